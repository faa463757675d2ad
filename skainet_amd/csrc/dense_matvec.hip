// Batch-1 product of a stacked dense matrix (bf16 or fp32 weights) with an fp32 vector: bound by the weight stream.
//
// The input is staged once per workgroup in LDS -- plain, divided group by group by its root mean square (the norm ahead
// of a layer), or with the split partials of an attention merged on the way in -- as two planes of float4 (even and odd
// fours of elements), so that the eight activations of a 16-byte piece of bf16 weights are two conflict-free 16-byte
// reads.  A wavefront takes a row at a time and walks on through the stacked rows; its next requests are under way while it
// multiplies, the first ones from before the staging.  Epilogue: bias and the operation
// of the segment, or the residual sum; a key projection also goes to its page of the cache.
#include "dense.h"

#include <algorithm>
#include <type_traits>

namespace {

typedef uint32_t u32x4 __attribute__((ext_vector_type(4)));

constexpr int kThreads = 1024, kWaves = kThreads / 64;
constexpr int kR = 1;  // rows per wavefront and turn (measured with two as well: slower at 1024 threads)
constexpr int kU = 4;  // 16-byte pieces per row and lane in flight, twice
constexpr int kMaxGroups = 256, kMaxMerge = 4096, kMaxSplits = 16;  // norm groups; heads x splits and splits of a merge

struct XPlanes {
    float4* even;
    float4* odd;
    __device__ __forceinline__ float4& quad(int q) const { return (q & 1) ? odd[q >> 1] : even[q >> 1]; }
    __device__ __forceinline__ float& at(int e) const { return reinterpret_cast<float*>(&quad(e >> 2))[e & 3]; }
};

__device__ __forceinline__ void stage_group_norm(const skn_matvec_src& s, const XPlanes& xs, float* red) {
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, quads = (s.k0 + 3) >> 2, gs = s.k0 / s.groups;
    // (pitches are multiples of 64 elements and their padding is zero: the last quad may be read whole)
    const bool few = s.groups <= 8 && (gs & 3) == 0;
    if (few) {
        float ss[8];
#pragma unroll
        for (int g = 0; g < 8; g++) ss[g] = 0.f;
        const float inv_quads = 4.0f / (float)gs;
        for (int q = tid; q < quads; q += kThreads) {
            const float4 v = reinterpret_cast<const float4*>(s.x0)[q];
            xs.quad(q) = v;
            const float d = (v.x * v.x + v.y * v.y) + (v.z * v.z + v.w * v.w);
            const int g = (int)(((float)q + 0.5f) * inv_quads);
#pragma unroll
            for (int i = 0; i < 8; i++) ss[i] += i == g ? d : 0.f;
        }
#pragma unroll
        for (int g = 0; g < 8; g++)
            if (g < s.groups) {
                const float t = wave_sum(ss[g]);
                if (lane == 0) red[g * kWaves + wave] = t;
            }
        __syncthreads();
        if (tid < s.groups) {
            float t = 0.f;
            for (int i = 0; i < kWaves; i++) t += red[tid * kWaves + i];
            red[8 * kWaves + tid] = 1.0f / sqrtf(t / (float)gs + s.eps);
        }
        __syncthreads();
        for (int q = tid; q < quads; q += kThreads) {
            const float r = red[8 * kWaves + (int)(((float)q + 0.5f) * inv_quads)];
            const float4 v = xs.quad(q), g = reinterpret_cast<const float4*>(s.norm_w)[q];
            xs.quad(q) = make_float4(v.x * r * g.x, v.y * r * g.y, v.z * r * g.z, v.w * r * g.w);
        }
        return;
    }
    for (int e = tid; e < s.k0; e += kThreads) xs.at(e) = s.x0[e];
    __syncthreads();
    for (int g = wave; g < s.groups; g += kWaves) {
        float ss = 0.f;
        for (int e = lane; e < gs; e += 64) {
            const float v = xs.at(g * gs + e);
            ss = fmaf(v, v, ss);
        }
        ss = wave_sum(ss);
        if (lane == 0) red[g] = 1.0f / sqrtf(ss / (float)gs + s.eps);
    }
    __syncthreads();
    for (int e = tid; e < s.k0; e += kThreads) xs.at(e) *= red[e / gs] * s.norm_w[e];
}

// the sum over the workgroup (a barrier inside; red: one float per wavefront, used once)
__device__ __forceinline__ float block_sum(float v, float* red) {
    v = wave_sum(v);
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
    __syncthreads();
    v = 0.f;
#pragma unroll
    for (int i = 0; i < kWaves; i++) v += red[i];
    return v;
}

// (pitches are multiples of 64 elements and their padding is zero, as in stage_group_norm; a thread's quads stay its own)
__device__ __forceinline__ void stage_add_norm(const skn_matvec_src& s, const XPlanes& xs, float* red) {
    const int tid = threadIdx.x, quads = (s.k0 + 3) >> 2;
    auto square = [](const float4& v) { return (v.x * v.x + v.y * v.y) + (v.z * v.z + v.w * v.w); };
    float ss = 0.f;
    for (int q = tid; q < quads; q += kThreads) {
        const float4 v = reinterpret_cast<const float4*>(s.add)[q];
        xs.quad(q) = v;
        ss += square(v);
    }
    const float ry = 1.0f / sqrtf(block_sum(ss, red) / (float)s.k0 + s.eps);
    ss = 0.f;
    for (int q = tid; q < quads; q += kThreads) {
        const float4 y = xs.quad(q), x = reinterpret_cast<const float4*>(s.x0)[q], g = reinterpret_cast<const float4*>(s.add_w)[q];
        const float4 v = make_float4(fmaf(y.x * ry, g.x, x.x), fmaf(y.y * ry, g.y, x.y), fmaf(y.z * ry, g.z, x.z), fmaf(y.w * ry, g.w, x.w));
        xs.quad(q) = v;
        if (blockIdx.x == 0) reinterpret_cast<float4*>(s.x_out)[q] = v;
        ss += square(v);
    }
    const float rx = 1.0f / sqrtf(block_sum(ss, red + kWaves) / (float)s.k0 + s.eps);
    for (int q = tid; q < quads; q += kThreads) {
        const float4 v = xs.quad(q), g = reinterpret_cast<const float4*>(s.norm_w)[q];
        xs.quad(q) = make_float4(v.x * rx * g.x, v.y * rx * g.y, v.z * rx * g.z, v.w * rx * g.w);
    }
}

// red: heads x splits weights
__device__ __forceinline__ void stage_merge(const skn_matvec_src& s, const XPlanes& xs, float* red) {
    const int tid = threadIdx.x;
    for (int h = tid; h < s.heads; h += kThreads) {
        float2 ml[kMaxSplits];  // (all requested before the first is used)
#pragma unroll
        for (int i = 0; i < kMaxSplits; i++) ml[i] = reinterpret_cast<const float2*>(s.ml)[min(i, s.splits - 1) * s.heads + h];
        float m = s.sink ? 0.f : -INFINITY;
#pragma unroll
        for (int i = 0; i < kMaxSplits; i++) m = fmaxf(m, ml[i].x);
        float l = s.sink ? __builtin_amdgcn_exp2f(-m) : 0.f;
#pragma unroll
        for (int i = 0; i < kMaxSplits; i++) {
            ml[i].x = i < s.splits ? __builtin_amdgcn_exp2f(ml[i].x - m) : 0.f;  // (an empty split: exp2(-inf) = 0)
            l = fmaf(ml[i].x, ml[i].y, l);
        }
        const float inv = 1.0f / l;
#pragma unroll
        for (int i = 0; i < kMaxSplits; i++)
            if (i < s.splits) red[h * s.splits + i] = ml[i].x * inv;
    }
    __syncthreads();
    if ((s.dim & 3) == 0) {
        const int dq = s.dim >> 2;
        const int64_t step = (int64_t)s.heads * s.dim_pad;
        for (int q = tid; q < s.heads * dq; q += kThreads) {
            const int h = q / dq, c = q - h * dq;
            const float* p = s.x0 + (int64_t)h * s.dim_pad + 4 * c;
            float4 a = make_float4(0.f, 0.f, 0.f, 0.f);
            for (int i0 = 0; i0 < s.splits; i0 += 8) {
                float4 v[8];
#pragma unroll
                for (int i = 0; i < 8; i++) v[i] = *reinterpret_cast<const float4*>(p + min(i0 + i, s.splits - 1) * step);
#pragma unroll
                for (int i = 0; i < 8; i++) {
                    const float f = i0 + i < s.splits ? red[h * s.splits + i0 + i] : 0.f;
                    a.x = fmaf(f, v[i].x, a.x), a.y = fmaf(f, v[i].y, a.y), a.z = fmaf(f, v[i].z, a.z), a.w = fmaf(f, v[i].w, a.w);
                }
            }
            if (s.gate) {
                const float4 g = reinterpret_cast<const float4*>(s.gate)[q];
                a.x *= g.x, a.y *= g.y, a.z *= g.z, a.w *= g.w;
            }
            xs.quad(q) = a;
        }
        return;
    }
    for (int e = tid; e < s.k0; e += kThreads) {
        const int h = e / s.dim, d = e - h * s.dim;
        float a = 0.f;
        for (int i = 0; i < s.splits; i++) a = fmaf(red[h * s.splits + i], s.x0[((int64_t)i * s.heads + h) * s.dim_pad + d], a);
        xs.at(e) = s.gate ? a * s.gate[e] : a;
    }
}

// W: uint16_t (bf16) or float.  LDS: two planes of `plane` float4, then the scratch of the staging.
template <typename W, int MODE>
__global__ __launch_bounds__(kThreads) void dense_matvec_kernel(const W* __restrict__ w, int rows, int k_pad, int plane,
                                                                const float* __restrict__ bias, const skn_matvec_src src,
                                                                const skn_dense_out out) {
    extern __shared__ __align__(16) float4 lds4[];
    constexpr int V = 16 / (int)sizeof(W);
    const XPlanes xs = {lds4, lds4 + plane};
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int pieces = k_pad / V;                           // 16-byte pieces of a row
    const int turns = (pieces + 64 * kU - 1) / (64 * kU);   // requests per row, kU pieces per lane each
    const int groups = (rows + kR - 1) / kR, stride = (int)gridDim.x * kWaves;
    int grp = (int)blockIdx.x * kWaves + wave, turn = 0;

    u32x4 cur[kR][kU], nxt[kR][kU];
    auto fetch = [&](u32x4(&buf)[kR][kU], int g, int t) __attribute__((always_inline)) {
#pragma unroll
        for (int r = 0; r < kR; r++) {
            const u32x4* row = reinterpret_cast<const u32x4*>(w + (int64_t)min(kR * g + r, rows - 1) * k_pad);
#pragma unroll
            for (int u = 0; u < kU; u++) buf[r][u] = row[min((t * kU + u) * 64 + lane, pieces - 1)];  // (past the end: times a zero of x)
        }
    };
    fetch(cur, min(grp, groups - 1), 0);

    // ---- staging ----
    if constexpr (MODE == SKN_XSRC_GROUP_NORM) stage_group_norm(src, xs, reinterpret_cast<float*>(lds4 + 2 * plane));
    else if constexpr (MODE == SKN_XSRC_ADD_NORM) stage_add_norm(src, xs, reinterpret_cast<float*>(lds4 + 2 * plane));
    else if constexpr (MODE == SKN_XSRC_MERGE) stage_merge(src, xs, reinterpret_cast<float*>(lds4 + 2 * plane));
    else {
        for (int q = tid; q < src.k0 >> 2; q += kThreads) xs.quad(q) = reinterpret_cast<const float4*>(src.x0)[q];
        for (int e = (src.k0 & ~3) + tid; e < src.k0; e += kThreads) xs.at(e) = src.x0[e];
    }
    if (src.x1) {
        for (int q = tid; q < src.k1 >> 2; q += kThreads) xs.quad((src.off1 >> 2) + q) = reinterpret_cast<const float4*>(src.x1)[q];
        for (int e = (src.k1 & ~3) + tid; e < src.k1; e += kThreads) xs.at(src.off1 + e) = src.x1[e];
    }
    {
        const int gap_end = src.x1 ? src.off1 : 8 * plane, tail = src.x1 ? src.off1 + src.k1 : 8 * plane;
        if constexpr (MODE == SKN_XSRC_GROUP_NORM || MODE == SKN_XSRC_ADD_NORM) __syncthreads();  // (its last quad may have been written past k0)
        for (int e = src.k0 + tid; e < gap_end; e += kThreads) xs.at(e) = 0.f;
        for (int e = tail + tid; e < 8 * plane; e += kThreads) xs.at(e) = 0.f;
    }
    __syncthreads();

    const float* bias_src = bias ? bias : reinterpret_cast<const float*>(w);
    const float* resid_src = out.nseg == 0 ? out.resid : reinterpret_cast<const float*>(w);
    const int resid_last = out.nseg == 0 ? out.resid_rows - 1 : rows - 1;
    int cache_page = 0, cache_slot = 0;
    if (out.cache_seg >= 0) {
        const int pos = *out.pos_dev;
        cache_page = out.page_table[pos / out.page_tokens];
        cache_slot = pos % out.page_tokens;
    }
    const int64_t mul_at = out.mul_seg >= 0 ? (int64_t)*out.mul_tokens * out.mul_ld + out.mul_col : 0;
    float acc[kR];
#pragma unroll
    for (int r = 0; r < kR; r++) acc[r] = 0.f;
    auto multiply = [&](const u32x4(&buf)[kR][kU], int t) __attribute__((always_inline)) {
#pragma unroll
        for (int u = 0; u < kU; u++) {
            const int p = (t * kU + u) * 64 + lane;
            if constexpr (sizeof(W) == 2) {
                const float4 a = xs.even[p], b = xs.odd[p];
                const float x[8] = {a.x, a.y, a.z, a.w, b.x, b.y, b.z, b.w};
#pragma unroll
                for (int r = 0; r < kR; r++)
#pragma unroll
                    for (int j = 0; j < 4; j++) {
                        const uint32_t d = buf[r][u][j];
                        acc[r] = fmaf(__uint_as_float(d << 16), x[2 * j], acc[r]);
                        acc[r] = fmaf(__uint_as_float(d & 0xFFFF0000u), x[2 * j + 1], acc[r]);
                    }
            } else {
                const float4 a = xs.quad(p);
                const float x[4] = {a.x, a.y, a.z, a.w};
#pragma unroll
                for (int r = 0; r < kR; r++)
#pragma unroll
                    for (int j = 0; j < 4; j++) {
                        const uint32_t d = buf[r][u][j];
                        acc[r] = fmaf(__uint_as_float(d), x[j], acc[r]);
                    }
            }
        }
    };
    auto store = [&](int g, float bias_v, float resid_v) __attribute__((always_inline)) {
        float z = 0.f;
#pragma unroll
        for (int r = 0; r < kR; r++) {
            const float t = wave_sum(acc[r]);
            z = lane == r ? t : z;
            acc[r] = 0.f;
        }
        const int row = kR * g + lane;
        if (lane >= kR || row >= rows) return;
        z += bias ? bias_v : 0.f;
        if (out.nseg == 0) {
            if (row < out.resid_rows) out.resid[row] = fmaf(out.mult, z, resid_v);
            return;
        }
        int si = -1;
        for (int q = 0; q < out.nseg; q++)
            if (kR * g >= out.seg[q].row0) si = q;  // (uniform: a group of rows does not cross segments)
        if (si < 0) return;
        const skn_dense_seg sg = out.seg[si];
        const int r = row - sg.row0;
        if (r >= sg.rows) return;
        z = skn_dense_op(sg.op, z, sg.p0, sg.p1);
        if (si == out.mul_seg) z *= skn_table_at(out.mul_table, out.mul_type, mul_at + r);
        if (sg.out_type == SKN_TYPE_F32) ((float*)sg.out)[r] = z;
        else ((uint16_t*)sg.out)[r] = skn_bf16_bits(z);
        if (si == out.cache_seg) {
            const int h = r / out.dim;
            const int64_t at = (((int64_t)cache_page * out.kv_heads + h) * out.page_tokens + cache_slot) * out.dim_pad + (r - h * out.dim);
            if (out.elem_type == SKN_TYPE_F32) ((float*)out.k_pool)[at] = z;
            else ((uint16_t*)out.k_pool)[at] = __half_as_ushort(__float2half_rn(z));
        }
    };
    // one turn on `buf` while the next turn's weights arrive in `other`
    auto step = [&](u32x4(&buf)[kR][kU], u32x4(&other)[kR][kU]) __attribute__((always_inline)) {
        const int g = grp, t = turn;
        // What the store will need is asked for ahead of the weights, or waiting for it would wait for them; every turn
        // and with whatever address there is (a row of w holds at least 128 bytes), so that the number of requests
        // outstanding is known.
        const int row = min(kR * g + (lane & (kR - 1)), rows - 1);
        float bias_v = bias_src[row], resid_v = resid_src[min(row, resid_last)];
        __builtin_amdgcn_sched_barrier(0);
        if (++turn == turns) turn = 0, grp += stride;
        fetch(other, min(grp, groups - 1), turn);  // (unconditional, so that the wait below is for a known number of newer requests)
        __builtin_amdgcn_sched_barrier(0);
        multiply(buf, t);
        asm volatile("" : "+v"(bias_v), "+v"(resid_v));  // (keeps the two requests where they are written)
        if (t == turns - 1 && g < groups) store(g, bias_v, resid_v);
        __builtin_amdgcn_sched_barrier(0);
    };
    while (grp < groups) {
        step(cur, nxt);
        step(nxt, cur);  // (past the last group: a repeat of its last rows, not stored)
    }
}

constexpr int kMaxLds = 160 * 1024;

template <typename W, int MODE>
int launch(skn_ctx* ctx, const skn_dense_mat& w, const skn_matvec_src& src, const skn_dense_out& out) {
    constexpr int V = 16 / (int)sizeof(W);
    const int chunk = 64 * kU * V;  // elements of a turn: the planes hold whole turns
    const int plane = (w.k_pad + chunk - 1) / chunk * chunk / 8;
    const size_t scratch = MODE == SKN_XSRC_GROUP_NORM || MODE == SKN_XSRC_ADD_NORM ? (kMaxGroups + 16 * kWaves) * 4 : MODE == SKN_XSRC_MERGE ? (size_t)src.heads * src.splits * 4 : 0;
    const size_t lds = (size_t)plane * 32 + scratch;
    SKN_REQUIRE(ctx, lds <= kMaxLds, SKN_ERR_SHAPE, "dense matvec: %d columns need %zu bytes of LDS (at most %d)", w.k_pad, lds, kMaxLds);
    // one workgroup per compute unit at most: its staging serves all the rows its wavefronts walk through
    const int groups = (w.rows + kR - 1) / kR, blocks = std::min((groups + kWaves - 1) / kWaves, ctx->compute_units);
    skn_launch(ctx, dense_matvec_kernel<W, MODE>, dim3((unsigned)blocks), dim3(kThreads), lds, (const W*)w.w, w.rows, w.k_pad, plane, w.bias, src, out);
    SKN_LAUNCH_CHECK(ctx);
    return SKN_OK;
}

template <typename W>
int launch_mode(skn_ctx* ctx, const skn_dense_mat& w, const skn_matvec_src& src, const skn_dense_out& out) {
    if (src.mode == SKN_XSRC_GROUP_NORM) return launch<W, SKN_XSRC_GROUP_NORM>(ctx, w, src, out);
    if (src.mode == SKN_XSRC_ADD_NORM) return launch<W, SKN_XSRC_ADD_NORM>(ctx, w, src, out);
    if (src.mode == SKN_XSRC_MERGE) return launch<W, SKN_XSRC_MERGE>(ctx, w, src, out);
    return launch<W, SKN_XSRC_PLAIN>(ctx, w, src, out);
}

template <typename W, int MODE>
int allow_lds(skn_ctx* ctx) {
    SKN_HIP(ctx, hipFuncSetAttribute((const void*)dense_matvec_kernel<W, MODE>, hipFuncAttributeMaxDynamicSharedMemorySize, kMaxLds));
    return SKN_OK;
}

int dense_matvec_init(skn_ctx* ctx) {
    SKN_TRY((allow_lds<uint16_t, SKN_XSRC_PLAIN>(ctx)));
    SKN_TRY((allow_lds<uint16_t, SKN_XSRC_GROUP_NORM>(ctx)));
    SKN_TRY((allow_lds<uint16_t, SKN_XSRC_ADD_NORM>(ctx)));
    SKN_TRY((allow_lds<uint16_t, SKN_XSRC_MERGE>(ctx)));
    SKN_TRY((allow_lds<float, SKN_XSRC_ADD_NORM>(ctx)));
    SKN_TRY((allow_lds<float, SKN_XSRC_PLAIN>(ctx)));
    SKN_TRY((allow_lds<float, SKN_XSRC_GROUP_NORM>(ctx)));
    return allow_lds<float, SKN_XSRC_MERGE>(ctx);
}
skn_family register_family(dense_matvec_init);

}  // namespace

int skn_dense_matvec(skn_ctx* ctx, const skn_dense_mat& w, const skn_matvec_src& src, const skn_dense_out& out) {
    SKN_REQUIRE(ctx, w.w && w.rows > 0 && w.k_pad > 0 && w.k_pad % kDenseColPad == 0 && ((uintptr_t)w.w & 15) == 0, SKN_ERR_ARG,
                "dense matvec: bad matrix (%d x %d)", w.rows, w.k_pad);
    SKN_REQUIRE(ctx, src.x0 && ((uintptr_t)src.x0 & 15) == 0 && src.k0 > 0 && src.k0 <= w.k_pad, SKN_ERR_ARG, "dense matvec: bad input");
    SKN_REQUIRE(ctx, !src.x1 || (src.off1 >= src.k0 && src.off1 % 4 == 0 && src.off1 + src.k1 <= w.k_pad && ((uintptr_t)src.x1 & 15) == 0), SKN_ERR_ARG,
                "dense matvec: bad second input");
    SKN_REQUIRE(ctx, src.mode != SKN_XSRC_GROUP_NORM || (src.norm_w && src.groups > 0 && src.groups <= kMaxGroups && src.k0 % src.groups == 0),
                SKN_ERR_SHAPE, "dense matvec: %d norm groups of %d columns (at most %d groups)", src.groups, src.k0, kMaxGroups);
    SKN_REQUIRE(ctx, src.mode != SKN_XSRC_ADD_NORM || (src.norm_w && src.add && src.add_w && src.x_out && src.x_out != src.x0), SKN_ERR_ARG,
                "dense matvec: a sum and norm without its vectors");
    SKN_REQUIRE(ctx, out.mul_seg < 0 || (out.mul_table && out.mul_tokens), SKN_ERR_ARG, "dense matvec: no table to multiply with");
    SKN_REQUIRE(ctx, src.mode != SKN_XSRC_MERGE || (src.ml && src.splits > 0 && src.splits <= kMaxSplits && src.heads * src.splits <= kMaxMerge && src.k0 == src.heads * src.dim &&
                                                     src.dim_pad % 4 == 0),
                SKN_ERR_SHAPE, "dense matvec: cannot merge %d heads x %d splits", src.heads, src.splits);
    SKN_REQUIRE(ctx, out.nseg >= 0 && out.nseg <= kDenseMaxSegs && (out.nseg > 0 || out.resid), SKN_ERR_ARG, "dense matvec: no output");
    if (w.type == SKN_TYPE_BF16) return launch_mode<uint16_t>(ctx, w, src, out);
    if (w.type == SKN_TYPE_F32) return launch_mode<float>(ctx, w, src, out);
    return skn_fail(ctx, SKN_ERR_TYPE, "dense matvec: weights of type %d (BF16 or F32)", w.type);
}
