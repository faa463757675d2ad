// Attention that streams cached rows: a row is spread over a group of lanes, every group owns a private softmax stream, nothing
// is staged and no barrier is met while rows stream.  What the kernels over shared, ranged and latent caches have in common, and the
// kernel of the latter two.
#pragma once
#include "dense.h"
#include "kv.h"

namespace {

typedef uint32_t u32x4 __attribute__((ext_vector_type(4)));
typedef _Float16 half2_t __attribute__((ext_vector_type(2)));

constexpr float kLog2e = 1.4426950408889634f;

template <typename E>
struct Row8;  // eight elements of a cached row
template <>
struct Row8<uint16_t> {
    u32x4 a;
    __device__ __forceinline__ void load(const uint16_t* p) { a = *reinterpret_cast<const u32x4*>(p); }
    __device__ __forceinline__ void get(float (&f)[8]) const {
#pragma unroll
        for (int j = 0; j < 4; j++) {
            const uint32_t w = a[j];  // (a bit cast applied directly to a vector element reads element 0)
            const half2_t h = __builtin_bit_cast(half2_t, w);
            f[2 * j] = (float)h.x;
            f[2 * j + 1] = (float)h.y;
        }
    }
};
template <>
struct Row8<float> {
    float4 a, b;
    __device__ __forceinline__ void load(const float* p) {
        a = *reinterpret_cast<const float4*>(p);
        b = *reinterpret_cast<const float4*>(p + 4);
    }
    __device__ __forceinline__ void get(float (&f)[8]) const {
        f[0] = a.x, f[1] = a.y, f[2] = a.z, f[3] = a.w, f[4] = b.x, f[5] = b.y, f[6] = b.z, f[7] = b.w;
    }
};

// the value of lane ^ OFF (8, 16 or 32), for sums and maxima over lanes that differ in that bit: f(v, other)
template <int OFF, typename F>
__device__ __forceinline__ float with_lane_xor(float v, F f) {
    if constexpr (OFF == 8) return f(v, __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), 0x128, 0xF, 0xF, true)));  // row rotated by 8
    else if constexpr (OFF == 16) {
        const auto r = __builtin_amdgcn_permlane16_swap(__float_as_uint(v), __float_as_uint(v), false, false);
        return f(__uint_as_float(r[0]), __uint_as_float(r[1]));
    } else {
        const auto r = __builtin_amdgcn_permlane32_swap(__float_as_uint(v), __float_as_uint(v), false, false);
        return f(__uint_as_float(r[0]), __uint_as_float(r[1]));
    }
}

// over the 64 / LPT groups of a wavefront
template <int LPT, typename F>
__device__ __forceinline__ float over_groups(float v, F f) {
    if constexpr (LPT <= 8) v = with_lane_xor<8>(v, f);
    if constexpr (LPT <= 16) v = with_lane_xor<16>(v, f);
    return with_lane_xor<32>(v, f);
}

// a value as a cache of this element type holds it
template <typename E>
__device__ __forceinline__ float as_cached(float v) {
    if constexpr (sizeof(E) == 4) return v;
    else return __half2float(__float2half_rn(v));
}
template <typename E>
__device__ __forceinline__ void store_cached(E* p, float v) {
    if constexpr (sizeof(E) == 4) *p = v;
    else *p = __half_as_ushort(__float2half_rn(v));
}

// ---- rows of a ranged or a latent cache ---------------------------------------------------------------------------------

struct StreamArgs {
    const void* k_pool;
    const void* v_pool;
    const int32_t* table;  // the sequence's row of the page table
    int page_tokens, pages_per_seq, n_head, kv_heads, kdim, vdim;
    float inv_page;
    float scale, softcap;
    skn_range range;
    int sink, n_splits;
    float* opart;
    float* ml;
    void* out;  // [row][ldo], vdim columns per head
    int ldo, out_type;
    const float* gate;  // [row][ldg] factors of the output, or null
    int ldg;
    const int32_t* state;  // a step's device scalars (context length at [2]), or null: row z sees first_ctx + z tokens
    int first_ctx;
    const float* q_prep;  // [row][head][width]
    // a fused step: raw projections and what is done to them
    const float* q;
    const float* k;
    const float* v;
    const float* q_norm;
    const float* k_norm;
    const double* freq;
    int rot_dims;
    float eps;
};

// scores are handled in units of log2 e
__device__ __forceinline__ float stream_score(const StreamArgs& p, float dot) {
    float s = dot * p.scale;
    if (p.softcap > 0.f) s = p.softcap * tanhf(s / p.softcap);
    return s * kLog2e;
}

enum { kStreamRows = 0, kStreamStep = 1, kStreamLatent = 2 };

template <int KIND>
constexpr int stream_threads() { return KIND == kStreamLatent ? 512 : 1024; }

// Rows of W = 8 LPT KP elements; lane c of a row's LPT lanes has the pieces of eight elements c, LPT + c, ..
// kStreamRows: keys and values apart, prepared queries.  kStreamStep: the same for one token, whose norms, rotation and cache rows
// are this launch's prologue, while the first rows are on their way; its own key and value enter at the merge.
// kStreamLatent: the first vdim elements of the key row are the value.
// grid (splits, query heads, query rows)
template <typename E, int LPT, int KP, int KIND>
__global__ __launch_bounds__(stream_threads<KIND>()) void stream_attn_kernel(const StreamArgs p) {
    constexpr int kThreads = stream_threads<KIND>(), kWaves = kThreads / 64, G = 64 / LPT, NS = kWaves * G, W = 8 * LPT * KP;
    constexpr int U = KIND == kStreamLatent ? (sizeof(E) == 4 || KP > 5 ? 1 : 2) : sizeof(E) == 4 ? 2 : 4;  // rows per stream in flight
    constexpr bool LATENT = KIND == kStreamLatent, STEP = KIND == kStreamStep;
    static_assert(LATENT || KP == 1, "one piece per lane for keys and values apart");
    __shared__ float so[kWaves][W];
    __shared__ float sm[kWaves], sl[kWaves];
    __shared__ __align__(16) float own[STEP ? 3 : 1][STEP ? W : 4];  // the token's own q, k, v
    __shared__ float own_score;
    const int split = blockIdx.x, h = blockIdx.y, row = blockIdx.z, per_kv = p.n_head / p.kv_heads, kvh = h / per_kv;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, c = lane % LPT, g = lane / LPT, stream = wave * G + g;
    constexpr int kOwn = STEP ? W / 64 : 1;
    float raw[kOwn];  // wavefronts 0, 1, 2: q, k, v
    if constexpr (STEP) {
        const float* src = wave == 0 ? p.q + h * p.kdim : wave == 1 ? p.k + kvh * p.kdim : p.v + kvh * p.vdim;
        const int dim = wave == 2 ? p.vdim : p.kdim;
#pragma unroll
        for (int j = 0; j < kOwn; j++) raw[j] = wave < 3 && lane + 64 * j < dim ? src[lane + 64 * j] : 0.f;
    }
    const int n = p.state ? p.state[2] : p.first_ctx + row;
    const int lo = p.range.first(n - 1), hi = STEP ? n - 1 : n;  // the cached rows
    const int per = ((hi - lo + p.n_splits - 1) / p.n_splits + NS - 1) / NS * NS;
    const int t_begin = lo + split * per, t_end = min(hi, t_begin + per);
    // 64 page ids from the first one on ride in a register
    const int page0 = t_begin < t_end ? (int)(((float)t_begin + 0.5f) * p.inv_page) : 0;
    const int my_page = p.table[min(page0 + lane, p.pages_per_seq - 1)];

    constexpr int VP = LATENT ? 1 : KP;
    struct Rows {
        Row8<E> k[U][KP], v[LATENT ? 1 : U][VP];
    };
    Rows cur, nxt;
    auto fetch = [&](Rows& r, int base) __attribute__((always_inline)) {
#pragma unroll
        for (int u = 0; u < U; u++) {
            const int t = min(base + u * NS + stream, t_end - 1);  // past the end: a valid row, masked below
            const int pi = (int)(((float)t + 0.5f) * p.inv_page), slot = t - pi * p.page_tokens;  // (exact below 2^22 tokens)
            int page = __shfl(my_page, (pi - page0) & 63, 64);
            if (pi - page0 >= 64) page = p.table[pi];
            const int64_t at = (((int64_t)page * (LATENT ? 1 : p.kv_heads) + (LATENT ? 0 : kvh)) * p.page_tokens + slot) * W + c * 8;
#pragma unroll
            for (int j = 0; j < KP; j++) r.k[u][j].load((const E*)p.k_pool + at + 8 * LPT * j);
            if constexpr (!LATENT) {
#pragma unroll
                for (int j = 0; j < KP; j++) r.v[u][j].load((const E*)p.v_pool + at + 8 * LPT * j);
            }
        }
    };
    if (t_begin < t_end) fetch(cur, t_begin);

    float qf[KP][8];
    if constexpr (STEP) {
        if (wave < 3) {
            float f = 1.f;
            const float* norm = wave == 0 ? p.q_norm : p.k_norm;
            if (wave < 2 && norm) {
                float ss = 0.f;
#pragma unroll
                for (int j = 0; j < kOwn; j++) ss = fmaf(raw[j], raw[j], ss);
                f = 1.0f / sqrtf(wave_sum(ss) / (float)p.kdim + p.eps);
            }
#pragma unroll
            for (int j = 0; j < kOwn; j++) {
                const int e = lane + 64 * j;
                own[wave][e] = wave < 2 ? raw[j] * f * (norm && e < p.kdim ? norm[e] : 1.f) : as_cached<E>(raw[j]);
            }
        }
        __syncthreads();
        const int half = p.rot_dims >> 1, i = tid & 511;
        if (i < half) {  // (threads 0 .. the query, threads 512 .. the key)
            float sn, cs;
            skn_rope_sincos_freq(n - 1, p.freq[i], &sn, &cs);
            float* x = own[tid >> 9];
            const float u = x[i], v = x[i + half];
            x[i] = u * cs - v * sn;
            x[i + half] = v * cs + u * sn;
        }
        __syncthreads();
        if (tid < W) own[1][tid] = as_cached<E>(own[1][tid]);
        if (split == 0 && h % per_kv == 0) {
            const int pi = (n - 1) / p.page_tokens;
            const int64_t at = (((int64_t)p.table[pi] * p.kv_heads + kvh) * p.page_tokens + (n - 1) - pi * p.page_tokens) * W;
            if (tid < p.kdim) store_cached((E*)p.k_pool + at + tid, own[1][tid]);  // (the same thread wrote it)
            if (tid < p.vdim) store_cached((E*)p.v_pool + at + tid, own[2][tid]);
        }
        const float4 a = *reinterpret_cast<const float4*>(&own[0][c * 8]), b = *reinterpret_cast<const float4*>(&own[0][c * 8 + 4]);
        qf[0][0] = a.x, qf[0][1] = a.y, qf[0][2] = a.z, qf[0][3] = a.w, qf[0][4] = b.x, qf[0][5] = b.y, qf[0][6] = b.z, qf[0][7] = b.w;
        __syncthreads();
        if (wave == 0) {
            float d = 0.f;
#pragma unroll
            for (int j = 0; j < kOwn; j++) d = fmaf(own[0][lane + 64 * j], own[1][lane + 64 * j], d);
            d = wave_sum(d);
            if (lane == 0) own_score = stream_score(p, d);  // (read behind the merge's barrier)
        }
    } else {
#pragma unroll
        for (int j = 0; j < KP; j++) {
            const float4* qp = reinterpret_cast<const float4*>(p.q_prep + ((int64_t)row * p.n_head + h) * W + 8 * (j * LPT + c));
            const float4 a = qp[0], b = qp[1];
            qf[j][0] = a.x, qf[j][1] = a.y, qf[j][2] = a.z, qf[j][3] = a.w, qf[j][4] = b.x, qf[j][5] = b.y, qf[j][6] = b.z, qf[j][7] = b.w;
        }
    }
    float o[KP][8], m_run = -INFINITY, l_run = 0.f;
#pragma unroll
    for (int j = 0; j < KP; j++)
#pragma unroll
        for (int e = 0; e < 8; e++) o[j][e] = 0.f;

    auto absorb = [&](const Rows& r, int base) __attribute__((always_inline)) {
        float sc[U];
        float m_new = m_run;
#pragma unroll
        for (int u = 0; u < U; u++) {
            float d = 0.f;
#pragma unroll
            for (int j = 0; j < KP; j++) {
                float kf[8];
                r.k[u][j].get(kf);
#pragma unroll
                for (int e = 0; e < 8; e++) d = fmaf(kf[e], qf[j][e], d);
            }
            d = lane_group_sum<LPT>(d);
            sc[u] = base + u * NS + stream < t_end ? stream_score(p, d) : -INFINITY;
            m_new = fmaxf(m_new, sc[u]);
        }
        const float m_safe = m_new == -INFINITY ? 0.f : m_new;  // keeps exp2(-inf - -inf) out of the arithmetic
        const float alpha = __builtin_amdgcn_exp2f(m_run - m_safe);
        float sum = 0.f;
#pragma unroll
        for (int u = 0; u < U; u++) sum += sc[u] = __builtin_amdgcn_exp2f(sc[u] - m_safe);
        l_run = fmaf(l_run, alpha, sum);
        m_run = m_new;
#pragma unroll
        for (int j = 0; j < KP; j++) {
#pragma unroll
            for (int e = 0; e < 8; e++) o[j][e] *= alpha;
#pragma unroll
            for (int u = 0; u < U; u++) {
                float vf[8];
                if constexpr (LATENT) r.k[u][j].get(vf);
                else r.v[u][j].get(vf);
#pragma unroll
                for (int e = 0; e < 8; e++) o[j][e] = fmaf(sc[u], vf[e], o[j][e]);
            }
        }
    };
    for (int base = t_begin; base < t_end; base += NS * U) {
        fetch(nxt, base + NS * U);
        absorb(cur, base);
        cur = nxt;
    }

    // the G streams of the wavefront (lanes with the same c hold the same elements), then the wavefronts through LDS
    const auto add = [](float a, float b) { return a + b; };
    const float mw = over_groups<LPT>(m_run, [](float a, float b) { return fmaxf(a, b); });
    const float f = __builtin_amdgcn_exp2f(m_run - (mw == -INFINITY ? 0.f : mw));  // (an empty stream: exp2(-inf) = 0)
    const float lw = over_groups<LPT>(l_run * f, add);
#pragma unroll
    for (int j = 0; j < KP; j++)
#pragma unroll
        for (int e = 0; e < 8; e++) {
            const float x = over_groups<LPT>(o[j][e] * f, add);
            if (g == 0) so[wave][8 * (j * LPT + c) + e] = x;
        }
    if (lane == 0) sm[wave] = mw, sl[wave] = lw;
    __syncthreads();
    const bool with_own = STEP && split == 0, with_sink = p.sink && p.n_splits == 1;
    for (int d = tid; d < W; d += kThreads) {
        float m = with_own ? own_score : -INFINITY, acc = 0.f, l = 0.f;
        if (with_sink) m = fmaxf(m, 0.f);
#pragma unroll
        for (int w = 0; w < kWaves; w++) m = fmaxf(m, sm[w]);
        const float m_safe = m == -INFINITY ? 0.f : m;
#pragma unroll
        for (int w = 0; w < kWaves; w++) {
            const float x = __builtin_amdgcn_exp2f(sm[w] - m_safe);
            acc = fmaf(x, so[w][d], acc);
            l = fmaf(x, sl[w], l);
        }
        if constexpr (STEP) {
            if (with_own) {
                const float x = __builtin_amdgcn_exp2f(own_score - m_safe);
                acc = fmaf(x, own[2][d], acc);
                l += x;
            }
        }
        if (p.n_splits > 1) {
            p.opart[((int64_t)split * p.n_head + h) * W + d] = acc;
            if (d == 0) p.ml[2 * (split * p.n_head + h)] = m, p.ml[2 * (split * p.n_head + h) + 1] = l;
        } else if (d < p.vdim) {
            if (with_sink) l += __builtin_amdgcn_exp2f(-m_safe);
            float v = acc / l;
            if (p.gate) v *= p.gate[(int64_t)row * p.ldg + h * p.vdim + d];
            const int64_t at = (int64_t)row * p.ldo + h * p.vdim + d;
            if (p.out_type == SKN_TYPE_F32) ((float*)p.out)[at] = v;
            else ((uint16_t*)p.out)[at] = skn_bf16_bits(v);
        }
    }
}

// what every launch sets
inline StreamArgs stream_args(const skn_kv* kv, int seq, int n_head) {
    StreamArgs a = {};
    a.k_pool = kv->k_pool;
    a.v_pool = kv->v_pool;
    a.table = kv->page_table_dev + (size_t)seq * kv->pages_per_seq;
    a.page_tokens = kv->page_tokens;
    a.pages_per_seq = kv->pages_per_seq;
    a.n_head = n_head;
    a.kv_heads = kv->n_head;
    a.kdim = kv->dim;
    a.vdim = kv->vdim;
    a.inv_page = 1.0f / (float)kv->page_tokens;
    a.n_splits = 1;
    return a;
}

}  // namespace
