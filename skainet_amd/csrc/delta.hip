// The generalized delta rule and the state it runs on (rstate.h).
//
// Everything here is fp32.  Value channels of a head are independent columns of its state, so a group of L lanes owns a
// column: eight key channels per lane, the column's two dot products (with k before, with r after the update) are sums over
// the L lanes by DPP, and the state never leaves the registers between two tokens.  Because u = k / |k|, the removal term
// is (a k / |k|^2) (k^T S): one vector b = a k / (sum k^2 + 1e-6) beside k serves it.
//
// Prompts take two launches.  delta_pack_kernel writes, per head and token, the five vectors k, w, b, r, v one after the
// other, padded to the lanes' channels (and tokens that change nothing up to whole blocks); delta_scan_kernel -- one small
// workgroup per head and run of columns -- has the next 20 KB block of that stream on its way into registers while it computes
// the tokens of the current one out of LDS, each token's vectors read one token ahead.  (Copied straight into LDS instead,
// the compiler puts a wait for the copy in front of the next LDS read.)  The tokens of a sequence are a chain; what is
// parallel are the heads and the columns.
// A decode step is one launch, one workgroup per head: the decay's low-rank product, the step, the head's norm and the gate.
#include "dense.h"
#include "rstate.h"

#include <algorithm>

namespace {

constexpr float kUnitEps = 1e-6f;

struct Vec8 {
    float v[8];
    __device__ __forceinline__ void load(const float* p) {
        const float4 a = *reinterpret_cast<const float4*>(p), b = *reinterpret_cast<const float4*>(p + 4);
        v[0] = a.x, v[1] = a.y, v[2] = a.z, v[3] = a.w, v[4] = b.x, v[5] = b.y, v[6] = b.z, v[7] = b.w;
    }
    __device__ __forceinline__ void store(float* p) const {
        *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
        *reinterpret_cast<float4*>(p + 4) = make_float4(v[4], v[5], v[6], v[7]);
    }
};

template <int L>
__device__ __forceinline__ float dot_over_lanes(const Vec8& a, const Vec8& s) {
    float x = a.v[0] * s.v[0], y = a.v[1] * s.v[1];
#pragma unroll
    for (int j = 2; j < 8; j += 2) x = fmaf(a.v[j], s.v[j], x), y = fmaf(a.v[j + 1], s.v[j + 1], y);
    return lane_group_sum<L>(x + y);
}

// one token on one column; returns the column's output
template <int L>
__device__ __forceinline__ float delta_column(Vec8& s, const Vec8& k, const Vec8& w, const Vec8& b, const Vec8& r, float v) {
    const float y = dot_over_lanes<L>(k, s);
#pragma unroll
    for (int j = 0; j < 8; j++) s.v[j] = fmaf(w.v[j], s.v[j], fmaf(k.v[j], v, -b.v[j] * y));
    return dot_over_lanes<L>(r, s);
}

constexpr int kVecs = 5;  // k, w, b, r, v

constexpr int kBlockFloats = kVecs * 1024;  // a block of the packed stream: 1024 / dim_pad tokens
constexpr int kTrash = 64;                  // floats behind the stream that lanes without a column store to

__host__ __device__ inline int block_tokens(int dim_pad) { return 1024 / dim_pad; }
__host__ __device__ inline int padded_tokens(int n, int dim_pad) { return (n + block_tokens(dim_pad) - 1) / block_tokens(dim_pad) * block_tokens(dim_pad); }

// one wavefront per (token, head); n_pad: tokens with those that only fill the last block (k = b = 0, w = 1)
__global__ __launch_bounds__(256) void delta_pack_kernel(const float* __restrict__ r, const float* __restrict__ k, const float* __restrict__ v,
                                                         const float* __restrict__ w, const float* __restrict__ a, int ld, int n, int n_pad, int heads,
                                                         int dim, int dim_pad, float* __restrict__ pack) {
    const int id = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
    if (id >= n_pad * heads) return;
    const int t = id / heads, h = id - t * heads;
    const int64_t at = (int64_t)min(t, n - 1) * ld + h * dim;
    float kk[4], ss = 0.f;
#pragma unroll
    for (int i = 0; i < 4; i++) {
        const int d = lane + 64 * i;
        kk[i] = d < dim ? k[at + d] : 0.f;
        ss = fmaf(kk[i], kk[i], ss);
    }
    const float inv = 1.0f / (wave_sum(ss) + kUnitEps);
    float* out = pack + ((int64_t)h * n_pad + t) * kVecs * dim_pad;
#pragma unroll
    for (int i = 0; i < 4; i++) {
        const int d = lane + 64 * i;
        if (d >= dim_pad) continue;
        const bool in = d < dim && t < n;
        out[d] = in ? kk[i] : 0.f;
        out[dim_pad + d] = in ? w[at + d] : 1.f;
        out[2 * dim_pad + d] = in ? a[at + d] * kk[i] * inv : 0.f;
        out[3 * dim_pad + d] = in ? r[at + d] : 0.f;
        out[4 * dim_pad + d] = in ? v[at + d] : 0.f;
    }
}

// grid (column runs, heads); NW wavefronts of 64 / L columns each
template <int L, int NW>
__global__ __launch_bounds__(64 * NW) void delta_scan_kernel(const float* __restrict__ pack, int n, int n_pad, int heads, int dim,
                                                             float* __restrict__ state, float* __restrict__ o, float* __restrict__ trash) {
    __shared__ __align__(16) float lds[2][kBlockFloats];
    constexpr int DP = 8 * L, C = 1024 / DP, kTurns = kBlockFloats / 4 / (64 * NW);  // float4 per thread and block
    static_assert(kTurns * 4 * 64 * NW == kBlockFloats, "a block is whole float4 per thread");
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, h = blockIdx.y;
    const int rl = lane & (L - 1);
    const int col = (blockIdx.x * NW + wave) * (64 / L) + lane / L;
    const bool live = col < dim;
    const int colc = min(col, dim - 1);
    float* sp = state + ((int64_t)h * dim + colc) * DP + 8 * rl;
    Vec8 s;
    s.load(sp);
    const float4* src = reinterpret_cast<const float4*>(pack + (int64_t)h * n_pad * kVecs * DP) + tid;
    const int blocks = n_pad / C;
    float4 ahead[kTurns];
#pragma unroll
    for (int i = 0; i < kTurns; i++) ahead[i] = src[i * 64 * NW];

    struct Token {
        Vec8 k, w, b, r;
        float v;
    };
    for (int blk = 0; blk < blocks; blk++) {
        // (this buffer was last read two blocks ago, and everyone has passed the barrier since)
        float4* dst = reinterpret_cast<float4*>(lds[blk & 1]) + tid;
#pragma unroll
        for (int i = 0; i < kTurns; i++) dst[i * 64 * NW] = ahead[i];
        const float4* next = src + (int64_t)min(blk + 1, blocks - 1) * (kBlockFloats / 4);
#pragma unroll
        for (int i = 0; i < kTurns; i++) ahead[i] = next[i * 64 * NW];
        __builtin_amdgcn_sched_barrier(0);
        asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");
        const float* base = lds[blk & 1];
        const int t0 = blk * C;
        auto read = [&](Token& x, int t) __attribute__((always_inline)) {
            const float* p = base + t * kVecs * DP;
            x.k.load(p + 8 * rl);
            x.w.load(p + DP + 8 * rl);
            x.b.load(p + 2 * DP + 8 * rl);
            x.r.load(p + 3 * DP + 8 * rl);
            x.v = p[4 * DP + colc];
        };
        Token even, odd;
        read(even, 0);
        constexpr int G = L < C ? L : C;  // the L lanes of a column keep the outputs of G tokens and store them together
        float keep = 0.f;
#pragma unroll
        for (int t = 0; t < C; t += 2) {
            read(odd, t + 1);
            __builtin_amdgcn_sched_barrier(0);
            const float o0 = delta_column<L>(s, even.k, even.w, even.b, even.r, even.v);
            keep = rl == t % G ? o0 : keep;
            if (t + 2 < C) read(even, t + 2);
            __builtin_amdgcn_sched_barrier(0);
            const float o1 = delta_column<L>(s, odd.k, odd.w, odd.b, odd.r, odd.v);
            keep = rl == t % G + 1 ? o1 : keep;
            if ((t + 2) % G == 0) {
                // (one store whatever the lane: a skipped one would leave the number of requests outstanding unknown, and
                // the wait for the next block would wait for every store)
                const int mine = t0 + t + 2 - G + rl;
                float* p = live && rl < G && mine < n ? o + ((int64_t)mine * heads + h) * dim + col : trash + lane;
                *p = keep;
            }
        }
    }
    if (live) s.store(sp);
}

// one wavefront per (token, head)
__global__ __launch_bounds__(256) void delta_gate_kernel(const float* __restrict__ o, const float* __restrict__ g, int ldg, const float* __restrict__ norm,
                                                         int n, int heads, int dim, float eps, void* __restrict__ y, int ldy, int y_type) {
    const int id = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
    if (id >= n * heads) return;
    const int t = id / heads, h = id - t * heads;
    const float* p = o + (int64_t)id * dim;
    float x[4], ss = 0.f;
#pragma unroll
    for (int i = 0; i < 4; i++) {
        const int d = lane + 64 * i;
        x[i] = d < dim ? p[d] : 0.f;
        ss = fmaf(x[i], x[i], ss);
    }
    const float inv = 1.0f / sqrtf(wave_sum(ss) / (float)dim + eps);
#pragma unroll
    for (int i = 0; i < 4; i++) {
        const int d = lane + 64 * i;
        if (d >= dim) continue;
        const float f = x[i] * inv * norm[h * dim + d] * g[(int64_t)t * ldg + h * dim + d];
        const int64_t at = (int64_t)t * ldy + h * dim + d;
        if (y_type == SKN_TYPE_F32) ((float*)y)[at] = f;
        else ((uint16_t*)y)[at] = skn_bf16_bits(f);
    }
}

// one workgroup of NW wavefronts per head
template <int L, int NW, typename W>
__global__ __launch_bounds__(64 * NW) void delta_step_kernel(const skn_delta_step p, int dim, float* __restrict__ state) {
    constexpr int DP = 8 * L, CW = 64 / L, kThreads = 64 * NW;  // columns per wavefront
    constexpr int kPasses = (DP + NW * CW - 1) / (NW * CW);
    __shared__ __align__(16) float vec[kVecs][DP];
    __shared__ float so[DP], red[NW];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, h = blockIdx.x, rl = lane & (L - 1);
    const int off = h * dim;
    // the state first: it does not wait for anything
    Vec8 s[kPasses];
    float* sp[kPasses];
#pragma unroll
    for (int i = 0; i < kPasses; i++) {
        const int col = (i * NW + wave) * CW + lane / L;
        sp[i] = state + ((int64_t)off + min(col, dim - 1)) * DP + 8 * rl;
        s[i].load(sp[i]);
    }
    // decay: eight lanes per key channel share its row of w2
    for (int d = tid >> 3; d < DP; d += kThreads / 8) {
        float z = 0.f;
        if (d < dim) {
            const W* row = (const W*)p.w2 + (int64_t)(off + d) * p.rank_pad;
            for (int i = tid & 7; i < p.rank; i += 8) {
                float f;
                if constexpr (sizeof(W) == 2) f = __uint_as_float((uint32_t)row[i] << 16);
                else f = row[i];
                z = fmaf(f, p.t[i], z);
            }
        }
        z = lane_group_sum<8>(z);
        if ((tid & 7) == 0) vec[1][d] = d < dim ? skn_dense_op(SKN_OP_DECAY, z + p.b2[off + d], 0.f, 0.f) : 0.f;
    }
    float ss = 0.f;
    for (int d = tid; d < DP; d += kThreads) {
        const float kk = d < dim ? p.k[off + d] : 0.f;
        ss = fmaf(kk, kk, ss);
        vec[0][d] = kk;
        vec[2][d] = d < dim ? p.a[off + d] * kk : 0.f;  // (times 1 / (sum k^2 + eps) below)
        vec[3][d] = d < dim ? p.r[off + d] : 0.f;
        vec[4][d] = d < dim ? p.v[off + d] : 0.f;
    }
    ss = wave_sum(ss);
    if (lane == 0) red[wave] = ss;
    __syncthreads();
    ss = 0.f;
#pragma unroll
    for (int i = 0; i < NW; i++) ss += red[i];
    const float inv_k = 1.0f / (ss + kUnitEps);
    Vec8 k, w, b, r;
    k.load(&vec[0][8 * rl]);
    w.load(&vec[1][8 * rl]);
    b.load(&vec[2][8 * rl]);
    r.load(&vec[3][8 * rl]);
#pragma unroll
    for (int j = 0; j < 8; j++) b.v[j] *= inv_k;
#pragma unroll
    for (int i = 0; i < kPasses; i++) {
        const int col = (i * NW + wave) * CW + lane / L;
        const float out = delta_column<L>(s[i], k, w, b, r, vec[4][min(col, DP - 1)]);
        if (col < dim) {
            s[i].store(sp[i]);
            if (rl == 0) so[col] = out;
        }
    }
    __syncthreads();
    ss = 0.f;
    for (int d = tid; d < dim; d += kThreads) ss = fmaf(so[d], so[d], ss);
    ss = wave_sum(ss);
    if (lane == 0) red[wave] = ss;
    __syncthreads();
    ss = 0.f;
#pragma unroll
    for (int i = 0; i < NW; i++) ss += red[i];
    const float inv = 1.0f / sqrtf(ss / (float)dim + p.eps);
    for (int d = tid; d < dim; d += kThreads) p.y[off + d] = so[d] * inv * p.norm[off + d] * p.g[off + d];
}

template <int L, int NW>
int launch_scan(skn_ctx* ctx, const skn_rstate* st, const float* pack, int n, float* state, float* o) {
    const int per_wg = NW * (64 / L), n_pad = padded_tokens(n, st->dim_pad);
    float* trash = const_cast<float*>(pack) + (size_t)n_pad * st->heads * kVecs * st->dim_pad;
    skn_launch(ctx, delta_scan_kernel<L, NW>, dim3((st->dim + per_wg - 1) / per_wg, st->heads), dim3(64 * NW), 0, pack, n, n_pad, st->heads, st->dim, state,
               o, trash);
    SKN_LAUNCH_CHECK(ctx);
    return SKN_OK;
}

template <int L, int NW>
int launch_step(skn_ctx* ctx, const skn_rstate* st, const skn_delta_step& p, float* state) {
    if (p.w2_type == SKN_TYPE_F32) skn_launch(ctx, delta_step_kernel<L, NW, float>, dim3(st->heads), dim3(64 * NW), 0, p, st->dim, state);
    else skn_launch(ctx, delta_step_kernel<L, NW, uint16_t>, dim3(st->heads), dim3(64 * NW), 0, p, st->dim, state);
    SKN_LAUNCH_CHECK(ctx);
    return SKN_OK;
}

template <int L>
int scan_waves(skn_ctx* ctx, const skn_rstate* st, const float* pack, int n, float* state, float* o) {
    // one wavefront per workgroup spreads the columns over the compute units; four share the copied stream when there
    // are more column runs than compute units
    const int runs = st->heads * ((st->dim * L + 63) / 64);
    if (runs > 2 * ctx->compute_units) return launch_scan<L, 4>(ctx, st, pack, n, state, o);
    if (runs > ctx->compute_units) return launch_scan<L, 2>(ctx, st, pack, n, state, o);
    return launch_scan<L, 1>(ctx, st, pack, n, state, o);
}

__global__ void fill_zero_kernel(float4* p, int64_t n) {
    const int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
    if (i < n) p[i] = make_float4(0.f, 0.f, 0.f, 0.f);
}

}  // namespace

size_t skn_delta_pack_floats(const skn_rstate* st, int n) {
    return (size_t)padded_tokens(n, st->dim_pad) * st->heads * kVecs * st->dim_pad + kTrash;
}

int skn_delta_rows(skn_ctx* ctx, skn_rstate* st, int seq, const float* r, const float* k, const float* v, const float* w, const float* a, int ld, int n,
                   float* pack, float* o) {
    SKN_REQUIRE(ctx, n > 0 && (int64_t)(n + 32) * st->heads < ((int64_t)1 << 31) - 4, SKN_ERR_SHAPE, "delta rule: %d tokens x %d heads", n, st->heads);
    const int n_pad = padded_tokens(n, st->dim_pad);
    skn_launch(ctx, delta_pack_kernel, dim3((unsigned)(((int64_t)n_pad * st->heads + 3) / 4)), dim3(256), 0, r, k, v, w, a, ld, n, n_pad, st->heads, st->dim,
               st->dim_pad, pack);
    SKN_LAUNCH_CHECK(ctx);
    float* s = st->seq_state(seq);
    switch (st->dim_pad) {
        case 32: return scan_waves<4>(ctx, st, pack, n, s, o);
        case 64: return scan_waves<8>(ctx, st, pack, n, s, o);
        case 128: return scan_waves<16>(ctx, st, pack, n, s, o);
        default: return scan_waves<32>(ctx, st, pack, n, s, o);
    }
}

int skn_delta_gate_rows(skn_ctx* ctx, const float* o, const float* g, int ldg, const float* norm, int n, int heads, int dim, float eps, void* y, int ldy,
                        int y_type) {
    skn_launch(ctx, delta_gate_kernel, dim3((unsigned)(((int64_t)n * heads + 3) / 4)), dim3(256), 0, o, g, ldg, norm, n, heads, dim, eps, y, ldy, y_type);
    SKN_LAUNCH_CHECK(ctx);
    return SKN_OK;
}

int skn_delta_step_launch(skn_ctx* ctx, skn_rstate* st, int seq, const skn_delta_step& p) {
    float* s = st->seq_state(seq);
    switch (st->dim_pad) {
        case 32: return launch_step<4, 2>(ctx, st, p, s);
        case 64: return launch_step<8, 8>(ctx, st, p, s);
        case 128: return launch_step<16, 16>(ctx, st, p, s);
        default: return launch_step<32, 16>(ctx, st, p, s);
    }
}

extern "C" {

int skn_rstate_create(skn_ctx* ctx, int n_seq, int heads, int dim, skn_rstate** out) {
    SKN_REQUIRE(nullptr, ctx != nullptr, SKN_ERR_ARG, "skn_rstate_create: ctx is null");
    SKN_REQUIRE(ctx, out != nullptr, SKN_ERR_ARG, "skn_rstate_create: out is null");
    *out = nullptr;
    SKN_REQUIRE(ctx, n_seq > 0 && heads > 0, SKN_ERR_ARG, "skn_rstate_create: sizes must be positive");
    SKN_REQUIRE(ctx, dim > 0 && dim <= 256, SKN_ERR_SHAPE, "skn_rstate_create: heads of %d channels (1 to 256)", dim);
    skn_rstate* st = new (std::nothrow) skn_rstate();
    SKN_REQUIRE(ctx, st != nullptr, SKN_ERR_OOM, "skn_rstate_create: host allocation failed");
    st->n_seq = n_seq;
    st->heads = heads;
    st->dim = dim;
    st->dim_pad = dim <= 32 ? 32 : dim <= 64 ? 64 : dim <= 128 ? 128 : 256;
    const size_t bytes = (size_t)n_seq * heads * dim * st->dim_pad * sizeof(float);
    hipError_t e = hipMalloc((void**)&st->s, bytes);
    if (e != hipSuccess) {
        (void)hipGetLastError();
        delete st;
        return skn_fail(ctx, SKN_ERR_OOM, "skn_rstate_create: %zu bytes: %s", bytes, hipGetErrorString(e));
    }
    *out = st;
    const int rc = skn_rstate_reset(ctx, st, -1);
    if (rc != SKN_OK) {
        skn_rstate_free(ctx, st);
        *out = nullptr;
    }
    return rc;
}

int skn_rstate_free(skn_ctx* ctx, skn_rstate* st) {
    SKN_REQUIRE(nullptr, ctx != nullptr, SKN_ERR_ARG, "skn_rstate_free: ctx is null");
    if (!st) return SKN_OK;
    (void)hipStreamSynchronize(ctx->stream);
    if (st->s) (void)hipFree(st->s);
    delete st;
    return SKN_OK;
}

int skn_rstate_reset(skn_ctx* ctx, skn_rstate* st, int seq) {
    SKN_REQUIRE(nullptr, ctx != nullptr, SKN_ERR_ARG, "skn_rstate_reset: ctx is null");
    SKN_REQUIRE(ctx, st != nullptr, SKN_ERR_ARG, "skn_rstate_reset: state is null");
    SKN_REQUIRE(ctx, seq >= -1 && seq < st->n_seq, SKN_ERR_RANGE, "skn_rstate_reset: sequence %d of %d", seq, st->n_seq);
    const int64_t quads = (int64_t)st->heads * st->dim * st->dim_pad / 4 * (seq < 0 ? st->n_seq : 1);
    skn_launch(ctx, fill_zero_kernel, dim3((unsigned)((quads + 255) / 256)), dim3(256), 0, (float4*)st->seq_state(seq < 0 ? 0 : seq), quads);
    SKN_LAUNCH_CHECK(ctx);
    return SKN_OK;
}

int skn_delta_rule(skn_ctx* ctx, skn_rstate* st, int seq, const float* r_dev, const float* k_dev, const float* v_dev, const float* w_dev,
                   const float* a_dev, int n, float* out_dev) {
    SKN_REQUIRE(nullptr, ctx != nullptr, SKN_ERR_ARG, "skn_delta_rule: ctx is null");
    SKN_REQUIRE(ctx, st && r_dev && k_dev && v_dev && w_dev && a_dev && out_dev, SKN_ERR_ARG, "skn_delta_rule: null pointer");
    SKN_REQUIRE(ctx, seq >= 0 && seq < st->n_seq && n > 0, SKN_ERR_RANGE, "skn_delta_rule: %d tokens of sequence %d of %d", n, seq, st->n_seq);
    float* pack = nullptr;
    SKN_HIP(ctx, hipMalloc((void**)&pack, skn_delta_pack_floats(st, n) * sizeof(float)));
    const int rc = skn_delta_rows(ctx, st, seq, r_dev, k_dev, v_dev, w_dev, a_dev, st->heads * st->dim, n, pack, out_dev);
    (void)hipStreamSynchronize(ctx->stream);
    (void)hipFree(pack);
    return rc;
}

}  // extern "C"
