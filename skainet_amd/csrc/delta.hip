// The generalized delta rule and the state it runs on (rstate.h).
//
// Everything here is fp32, the matrix instructions (v_mfma_f32_16x16x4_f32) included.  Value channels of a head are independent
// columns of its state.  Because u = k / |k|, the removal term is (a k / |k|^2) (k^T S): one vector b = a k / (sum k^2 + 1e-6)
// beside k serves it.
//
// Prompts take two launches, and sixteen tokens (a chunk) are one step of the chain.  With W(s, t) the product of the decays of
// tokens s .. t of the chunk, S the state before it and y_t = k_t^T S_{t-1} what k_t reads,
//   (I + beta) Y = K0 S + alpha V,    K0_t = k_t W(0, t-1),   alpha_ts, beta_ts = k_t^T W(s+1, t-1) {k_s, b_s} for s < t
//   O = R0 S + gamma V - delta Y,     R0_t = r_t W(0, t),     gamma_ts, delta_ts = r_t^T W(s+1, t) {k_s, b_s} for s <= t
//   S' = W(0, 15) S + sum_s k_s W(s+1, 15) v_s - b_s W(s+1, 15) y_s
// delta_chunk_kernel -- one wavefront per chunk and head, all chunks at once, since none of it depends on the state -- forms the
// four triangles on the matrix cores, solves with I + beta, and leaves
//   Y = K1 S + A1 V,  O = R1 S + G1 V     (K1 = (I + beta)^-1 K0, A1 = (I + beta)^-1 alpha, R1 = R0 - delta K1, G1 = gamma - delta A1)
// as operands in the order in which the matrix instructions take them.  delta_scan_kernel then walks the chunks with one
// wavefront per head and sixteen columns, its part of S in accumulator layout -- which is also the layout of a column operand,
// so S and Y are multiplied as they stand -- and no LDS, no barrier: a chunk's operands are coalesced loads one chunk ahead.
// (Decays enter the triangles as ratios of products over at most sixteen tokens: any decay from 0.01 to 1 is safe in fp32.)
// A decode step is one launch, one workgroup per head: the decay's low-rank product, the step, the head's norm and the gate.
#include "delta.h"
#include "dense.h"
#include "rstate.h"

#include <algorithm>

namespace {

// one token on one column; returns the column's output
template <int L>
__device__ __forceinline__ float delta_column(Vec8& s, const Vec8& k, const Vec8& w, const Vec8& b, const Vec8& r, float v) {
    const float y = dot_over_lanes<L>(k, s);
#pragma unroll
    for (int j = 0; j < 8; j++) s.v[j] = fmaf(w.v[j], s.v[j], fmaf(k.v[j], v, -b.v[j] * y));
    return dot_over_lanes<L>(r, s);
}

constexpr int kTrash = 64;  // floats behind the operands that take the outputs of tokens past the end

// Operands of a chunk and head, in floats from its start.  Row operands (K1, R1: [token][channel], in tiles of 16 channels;
// A1, G1: [token][token]): lane 16 q + t holds elements 4 q .. 4 q + 3 of row t.  kT, bT ([channel][token], b negated) and V
// ([token][column] as a column operand): lane 16 q + c holds tokens 4 q .. 4 q + 3 of channel (column) c of the tile.
__host__ __device__ constexpr int off_k1(int) { return 0; }
__host__ __device__ constexpr int off_r1(int dp) { return 16 * dp; }
__host__ __device__ constexpr int off_kt(int dp) { return 32 * dp; }
__host__ __device__ constexpr int off_bt(int dp) { return 48 * dp; }
__host__ __device__ constexpr int off_v(int dp) { return 64 * dp; }
__host__ __device__ constexpr int off_a1(int dp) { return 80 * dp; }
__host__ __device__ constexpr int off_g1(int dp) { return 80 * dp + 256; }
__host__ __device__ constexpr int off_w(int dp) { return 80 * dp + 512; }
__host__ __device__ constexpr int chunk_floats(int dp) { return 81 * dp + 512; }

// N sums over the wavefront, step by step for all of them
template <int N>
__device__ __forceinline__ void wave_sums(float (&x)[N]) {
#pragma unroll
    for (int i = 0; i < N; i++) x[i] = lane_group_sum<16>(x[i]);
#pragma unroll
    for (int i = 0; i < N; i++) {
        const auto r = __builtin_amdgcn_permlane16_swap(__float_as_uint(x[i]), __float_as_uint(x[i]), false, false);
        x[i] = __uint_as_float(r[0]) + __uint_as_float(r[1]);
    }
#pragma unroll
    for (int i = 0; i < N; i++) {
        const auto r = __builtin_amdgcn_permlane32_swap(__float_as_uint(x[i]), __float_as_uint(x[i]), false, false);
        x[i] = __uint_as_float(r[0]) + __uint_as_float(r[1]);
    }
}

// x_t = rhs_t - sum_{s < t} beta_ts x_s, then z_t - sum_{s <= t} delta_ts x_s, for this lane's column; rows of rhs and z at
// pitch, replaced by the results
__device__ __forceinline__ void solve_column(float* rhs, float* z, int pitch, const float (*beta)[20], const float (*delta)[20]) {
    float x[kChunk];
#pragma unroll
    for (int t = 0; t < kChunk; t++) {
        x[t] = rhs[t * pitch];
#pragma unroll
        for (int s = 0; s < t; s++) x[t] = fmaf(-beta[t][s], x[s], x[t]);
        rhs[t * pitch] = x[t];
    }
#pragma unroll
    for (int t = 0; t < kChunk; t++) {
        float o = z[t * pitch];
#pragma unroll
        for (int s = 0; s <= t; s++) o = fmaf(-delta[t][s], x[s], o);
        z[t * pitch] = o;
    }
}

// one wavefront per (chunk, head); tokens past n change nothing (k = b = r = v = 0, decay 1)
template <int DP>
__global__ __launch_bounds__(64) void delta_chunk_kernel(const float* __restrict__ r, const float* __restrict__ k, const float* __restrict__ v,
                                                         const float* __restrict__ w, const float* __restrict__ a, int ld, int n, int heads, int dim,
                                                         float* __restrict__ ops) {
    constexpr int kPitch = DP + 4, kSets = (DP + 63) / 64, kTiles = DP / 16;
    __shared__ __align__(16) float row[4][kChunk * kPitch];  // K0 then K1, R0 then R1, k / W, b / W
    __shared__ __align__(16) float tri[4][kChunk][20];       // alpha then A1, gamma then G1, beta, delta
    const int lane = threadIdx.x, chunk = blockIdx.x, h = blockIdx.y, chunks = gridDim.x, t0 = chunk * kChunk;
    float* out = ops + ((int64_t)h * chunks + chunk) * chunk_floats(DP);
    float inv[kChunk];
#pragma unroll
    for (int t = 0; t < kChunk; t++) {
        inv[t] = 0.f;
        const float* kr = k + (int64_t)min(t0 + t, n - 1) * ld + h * dim;
#pragma unroll
        for (int i = 0; i < kSets; i++) {
            const float x = lane + 64 * i < dim ? kr[lane + 64 * i] : 0.f;
            inv[t] = fmaf(x, x, inv[t]);
        }
    }
    wave_sums<kChunk>(inv);
#pragma unroll
    for (int t = 0; t < kChunk; t++) inv[t] = 1.0f / (inv[t] + kUnitEps);

#pragma unroll 1
    for (int i = 0; i < kSets; i++) {
        const int d = lane + 64 * i;
        if (d >= DP) continue;
        float kk[kChunk], bb[kChunk], vv[kChunk], upto = 1.f;  // upto: W(0, t)
#pragma unroll
        for (int t = 0; t < kChunk; t++) {
            const bool in = d < dim && t0 + t < n;
            const int64_t at = (int64_t)min(t0 + t, n - 1) * ld + h * dim + min(d, dim - 1);
            const float kt = in ? k[at] : 0.f, wt = in ? w[at] : 1.f, bt = in ? a[at] * kt * inv[t] : 0.f, rt = in ? r[at] : 0.f;
            vv[t] = in ? v[at] : 0.f;
            row[0][t * kPitch + d] = kt * upto;
            upto *= wt;
            row[1][t * kPitch + d] = rt * upto;
            const float rec = 1.0f / upto;
            kk[t] = kt * rec;
            bb[t] = bt * rec;
            row[2][t * kPitch + d] = kk[t];
            row[3][t * kPitch + d] = bb[t];
        }
        out[off_w(DP) + d] = upto;
        // tile d / 16, lane 16 q + d % 16
        float* frag = out + ((d >> 4) * 64 + (d & 15)) * 4;
#pragma unroll
        for (int q = 0; q < 4; q++) {
            const f32x4 x = {kk[4 * q] * upto, kk[4 * q + 1] * upto, kk[4 * q + 2] * upto, kk[4 * q + 3] * upto};
            const f32x4 y = {-bb[4 * q] * upto, -bb[4 * q + 1] * upto, -bb[4 * q + 2] * upto, -bb[4 * q + 3] * upto};
            const f32x4 z = {vv[4 * q], vv[4 * q + 1], vv[4 * q + 2], vv[4 * q + 3]};
            *reinterpret_cast<f32x4*>(frag + off_kt(DP) + 64 * q) = x;
            *reinterpret_cast<f32x4*>(frag + off_bt(DP) + 64 * q) = y;
            *reinterpret_cast<f32x4*>(frag + off_v(DP) + 64 * q) = z;
        }
    }
    __syncthreads();
    // the triangles: rows K0, R0 times columns k / W, b / W
    const int t16 = lane & 15, q4 = lane >> 4;
    f32x4 g[4];  // alpha, gamma, beta, delta
#pragma unroll
    for (int i = 0; i < 4; i++) g[i] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 2
    for (int c = 0; c < kTiles; c++) {
        const int at = t16 * kPitch + 16 * c + 4 * q4;
        const f32x4 k0 = load4(&row[0][at]), r0 = load4(&row[1][at]), kw = load4(&row[2][at]), bw = load4(&row[3][at]);
#pragma unroll
        for (int e = 0; e < 4; e++) {
            g[0] = mma(k0[e], kw[e], g[0]);
            g[1] = mma(r0[e], kw[e], g[1]);
            g[2] = mma(k0[e], bw[e], g[2]);
            g[3] = mma(r0[e], bw[e], g[3]);
        }
    }
#pragma unroll
    for (int e = 0; e < 4; e++) {
        const int t = 4 * q4 + e, s = t16;
        tri[0][t][s] = s < t ? g[0][e] : 0.f;
        tri[1][t][s] = s <= t ? g[1][e] : 0.f;
        tri[2][t][s] = s < t ? g[2][e] : 0.f;
        tri[3][t][s] = s <= t ? g[3][e] : 0.f;
    }
    __syncthreads();
#pragma unroll 1
    for (int i = 0; i < kSets; i++) {
        const int d = lane + 64 * i;
        if (d < DP) solve_column(&row[0][d], &row[1][d], kPitch, tri[2], tri[3]);
    }
    if (lane < kChunk) solve_column(&tri[0][0][lane], &tri[1][0][lane], 20, tri[2], tri[3]);
    __syncthreads();
#pragma unroll 2
    for (int c = 0; c < kTiles; c++) {
        *reinterpret_cast<f32x4*>(out + off_k1(DP) + (c * 64 + lane) * 4) = load4(&row[0][t16 * kPitch + 16 * c + 4 * q4]);
        *reinterpret_cast<f32x4*>(out + off_r1(DP) + (c * 64 + lane) * 4) = load4(&row[1][t16 * kPitch + 16 * c + 4 * q4]);
    }
    *reinterpret_cast<f32x4*>(out + off_a1(DP) + lane * 4) = load4(&tri[0][t16][4 * q4]);
    *reinterpret_cast<f32x4*>(out + off_g1(DP) + lane * 4) = load4(&tri[1][t16][4 * q4]);
}

template <int DP>
struct ChunkOps {
    static constexpr int kTiles = DP / 16;
    f32x4 k1[kTiles], r1[kTiles], kt[kTiles], bt[kTiles], w[kTiles], v, a1, g1;
    __device__ __forceinline__ void load(const float* p, int lane, int tile) {
#pragma unroll
        for (int j = 0; j < kTiles; j++) {
            k1[j] = load4(p + off_k1(DP) + (j * 64 + lane) * 4);
            r1[j] = load4(p + off_r1(DP) + (j * 64 + lane) * 4);
        }
        v = load4(p + off_v(DP) + (tile * 64 + lane) * 4);
        a1 = load4(p + off_a1(DP) + lane * 4);
        g1 = load4(p + off_g1(DP) + lane * 4);
#pragma unroll
        for (int j = 0; j < kTiles; j++) {
            kt[j] = load4(p + off_kt(DP) + (j * 64 + lane) * 4);
            bt[j] = load4(p + off_bt(DP) + (j * 64 + lane) * 4);
            w[j] = load4(p + off_w(DP) + 16 * j + 4 * (lane >> 4));
        }
    }
};

// One wavefront per head and tile of sixteen columns.  The wavefronts of a head are on one XCD (blockIdx % 8): they read the
// same operands, which then come from memory once.
template <int DP>
__global__ __launch_bounds__(64) void delta_scan_kernel(const float* __restrict__ ops, int n, int chunks, int heads, int dim, float* __restrict__ state,
                                                        float* __restrict__ o, float* __restrict__ trash) {
    constexpr int kTiles = DP / 16;
    const int lane = threadIdx.x, tiles = (dim + 15) / 16, turn = (int)(blockIdx.x >> 3), h = (int)(blockIdx.x & 7) + 8 * (turn / tiles), tile = turn % tiles;
    if (h >= heads) return;
    // (lanes beyond the last column compute along on zeros of V and store nothing)
    const int col = 16 * tile + (lane & 15);
    const bool live = col < dim;
    float* sp = state + ((int64_t)h * dim + min(col, dim - 1)) * DP + 4 * (lane >> 4);
    f32x4 s[kTiles];
#pragma unroll
    for (int j = 0; j < kTiles; j++) s[j] = load4(sp + 16 * j);
    const float* src = ops + (int64_t)h * chunks * chunk_floats(DP);

    auto step = [&](const ChunkOps<DP>& x, int chunk) __attribute__((always_inline)) {
        f32x4 y = {0.f, 0.f, 0.f, 0.f}, z = y;
#pragma unroll
        for (int e = 0; e < 4; e++) y = mma(x.a1[e], x.v[e], y), z = mma(x.g1[e], x.v[e], z);
#pragma unroll
        for (int j = 0; j < kTiles; j++)
#pragma unroll
            for (int e = 0; e < 4; e++) y = mma(x.k1[j][e], s[j][e], y), z = mma(x.r1[j][e], s[j][e], z);
#pragma unroll
        for (int j = 0; j < kTiles; j++) s[j] *= x.w[j];
#pragma unroll
        for (int e = 0; e < 4; e++)
#pragma unroll
            for (int j = 0; j < kTiles; j++) s[j] = mma(x.kt[j][e], x.v[e], s[j]);
#pragma unroll
        for (int e = 0; e < 4; e++)
#pragma unroll
            for (int j = 0; j < kTiles; j++) s[j] = mma(x.bt[j][e], y[e], s[j]);
        // (one store per token whatever the lane: a skipped one would leave the number of requests outstanding unknown, and
        // the wait for the next chunk's operands would wait for the stores)
#pragma unroll
        for (int e = 0; e < 4; e++) {
            const int t = chunk * kChunk + 4 * (lane >> 4) + e;
            float* dst = live && t < n ? o + ((int64_t)t * heads + h) * dim + col : trash + lane;
            *dst = z[e];
        }
    };
    ChunkOps<DP> even;
    if constexpr (DP <= 128) {
        ChunkOps<DP> odd;
        even.load(src, lane, tile);
        for (int c = 0; c < chunks; c += 2) {
            odd.load(src + (int64_t)min(c + 1, chunks - 1) * chunk_floats(DP), lane, tile);
            __builtin_amdgcn_sched_barrier(0);
            step(even, c);
            if (c + 1 == chunks) break;
            even.load(src + (int64_t)min(c + 2, chunks - 1) * chunk_floats(DP), lane, tile);
            __builtin_amdgcn_sched_barrier(0);
            step(odd, c + 1);
        }
    } else {
        for (int c = 0; c < chunks; c++) {
            even.load(src + (int64_t)c * chunk_floats(DP), lane, tile);
            step(even, c);
        }
    }
    if (live) {
#pragma unroll
        for (int j = 0; j < kTiles; j++) *reinterpret_cast<f32x4*>(sp + 16 * j) = s[j];
    }
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
    __shared__ __align__(16) float vec[5][DP];  // k, w, b, r, v
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

template <int DP>
int launch_rows(skn_ctx* ctx, const skn_rstate* st, const float* r, const float* k, const float* v, const float* w, const float* a, int ld, int n, float* ops,
                float* state, float* o) {
    const int chunks = (n + kChunk - 1) / kChunk, tiles = (st->dim + 15) / 16;
    skn_launch(ctx, delta_chunk_kernel<DP>, dim3(chunks, st->heads), dim3(64), 0, r, k, v, w, a, ld, n, st->heads, st->dim, ops);
    SKN_LAUNCH_CHECK(ctx);
    float* trash = ops + (size_t)chunks * st->heads * chunk_floats(DP);
    skn_launch(ctx, delta_scan_kernel<DP>, dim3((unsigned)((st->heads + 7) / 8 * 8 * tiles)), dim3(64), 0, (const float*)ops, n, chunks, st->heads, st->dim, state, o,
               trash);
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

__global__ void fill_zero_kernel(float* p, int64_t n) {
    const int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
    if (i < n) p[i] = 0.f;
}

}  // namespace

size_t skn_delta_pack_floats(const skn_rstate* st, int n) {
    return (size_t)((n + kChunk - 1) / kChunk) * st->heads * chunk_floats(st->dim_pad) + kTrash;
}

int skn_delta_rows(skn_ctx* ctx, skn_rstate* st, int seq, const float* r, const float* k, const float* v, const float* w, const float* a, int ld, int n,
                   float* pack, float* o) {
    SKN_REQUIRE(ctx, n > 0 && st->heads <= 65535, SKN_ERR_SHAPE, "delta rule: %d tokens x %d heads", n, st->heads);
    float* s = st->seq_state(seq);
    switch (st->dim_pad) {
        case 32: return launch_rows<32>(ctx, st, r, k, v, w, a, ld, n, pack, s, o);
        case 64: return launch_rows<64>(ctx, st, r, k, v, w, a, ld, n, pack, s, o);
        case 128: return launch_rows<128>(ctx, st, r, k, v, w, a, ld, n, pack, s, o);
        default: return launch_rows<256>(ctx, st, r, k, v, w, a, ld, n, pack, s, o);
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

static int rstate_create(skn_ctx* ctx, int n_seq, int heads, int kv_heads, int dim, int vdim, int taps, skn_rstate** out) {
    SKN_REQUIRE(nullptr, ctx != nullptr, SKN_ERR_ARG, "skn_rstate_create: ctx is null");
    SKN_REQUIRE(ctx, out != nullptr, SKN_ERR_ARG, "skn_rstate_create: out is null");
    *out = nullptr;
    SKN_REQUIRE(ctx, n_seq > 0 && heads > 0, SKN_ERR_ARG, "skn_rstate_create: sizes must be positive");
    SKN_REQUIRE(ctx, dim > 0 && dim <= 256 && vdim > 0 && vdim <= 256, SKN_ERR_SHAPE, "skn_rstate_create: heads of %d and %d channels (1 to 256)", dim, vdim);
    skn_rstate* st = new (std::nothrow) skn_rstate();
    SKN_REQUIRE(ctx, st != nullptr, SKN_ERR_OOM, "skn_rstate_create: host allocation failed");
    st->n_seq = n_seq;
    st->heads = heads;
    st->dim = dim;
    st->vdim = vdim;
    st->dim_pad = dim <= 32 ? 32 : dim <= 64 ? 64 : dim <= 128 ? 128 : 256;
    st->kv_heads = kv_heads;
    st->taps = taps;
    st->channels = 2 * kv_heads * dim + heads * vdim;
    st->pos.assign(n_seq, 0);
    const size_t bytes = (size_t)n_seq * heads * vdim * st->dim_pad * sizeof(float);
    hipError_t e = hipMalloc((void**)&st->s, bytes);
    if (e == hipSuccess && taps > 0) e = hipMalloc((void**)&st->conv, (size_t)n_seq * taps * st->channels * sizeof(float));
    if (e != hipSuccess) {
        (void)hipGetLastError();
        if (st->s) (void)hipFree(st->s);
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

int skn_rstate_create(skn_ctx* ctx, int n_seq, int heads, int dim, skn_rstate** out) {
    return rstate_create(ctx, n_seq, heads, 0, dim, dim, 0, out);
}

int skn_rstate_create_conv(skn_ctx* ctx, int n_seq, int heads, int kv_heads, int dim, int vdim, int taps, skn_rstate** out) {
    SKN_REQUIRE(nullptr, ctx != nullptr, SKN_ERR_ARG, "skn_rstate_create_conv: ctx is null");
    SKN_REQUIRE(ctx, heads > 0 && kv_heads > 0 && heads % kv_heads == 0, SKN_ERR_SHAPE, "skn_rstate_create_conv: kv_heads (%d) must divide heads (%d)", kv_heads, heads);
    SKN_REQUIRE(ctx, taps >= 1 && taps <= 8, SKN_ERR_SHAPE, "skn_rstate_create_conv: convolutions of %d taps (1 to 8)", taps);
    return rstate_create(ctx, n_seq, heads, kv_heads, dim, vdim, taps, out);
}

int skn_rstate_free(skn_ctx* ctx, skn_rstate* st) {
    SKN_REQUIRE(nullptr, ctx != nullptr, SKN_ERR_ARG, "skn_rstate_free: ctx is null");
    if (!st) return SKN_OK;
    (void)hipStreamSynchronize(ctx->stream);
    if (st->s) (void)hipFree(st->s);
    if (st->conv) (void)hipFree(st->conv);
    delete st;
    return SKN_OK;
}

int skn_rstate_reset(skn_ctx* ctx, skn_rstate* st, int seq) {
    SKN_REQUIRE(nullptr, ctx != nullptr, SKN_ERR_ARG, "skn_rstate_reset: ctx is null");
    SKN_REQUIRE(ctx, st != nullptr, SKN_ERR_ARG, "skn_rstate_reset: state is null");
    SKN_REQUIRE(ctx, seq >= -1 && seq < st->n_seq, SKN_ERR_RANGE, "skn_rstate_reset: sequence %d of %d", seq, st->n_seq);
    const int first = seq < 0 ? 0 : seq, count = seq < 0 ? st->n_seq : 1;
    const int64_t n = (int64_t)st->heads * st->vdim * st->dim_pad * count, m = (int64_t)st->taps * st->channels * count;
    skn_launch(ctx, fill_zero_kernel, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, st->seq_state(first), n);
    SKN_LAUNCH_CHECK(ctx);
    if (m > 0) {
        skn_launch(ctx, fill_zero_kernel, dim3((unsigned)((m + 255) / 256)), dim3(256), 0, st->seq_conv(first), m);
        SKN_LAUNCH_CHECK(ctx);
    }
    std::fill(st->pos.begin() + first, st->pos.begin() + first + count, 0);
    return SKN_OK;
}

int skn_delta_rule(skn_ctx* ctx, skn_rstate* st, int seq, const float* r_dev, const float* k_dev, const float* v_dev, const float* w_dev,
                   const float* a_dev, int n, float* out_dev) {
    SKN_REQUIRE(nullptr, ctx != nullptr, SKN_ERR_ARG, "skn_delta_rule: ctx is null");
    SKN_REQUIRE(ctx, st && r_dev && k_dev && v_dev && w_dev && a_dev && out_dev, SKN_ERR_ARG, "skn_delta_rule: null pointer");
    SKN_REQUIRE(ctx, seq >= 0 && seq < st->n_seq && n > 0, SKN_ERR_RANGE, "skn_delta_rule: %d tokens of sequence %d of %d", n, seq, st->n_seq);
    SKN_REQUIRE(ctx, st->taps == 0, SKN_ERR_STATE, "skn_delta_rule: the state has convolutions (skn_gated_delta)");
    float* pack = nullptr;
    SKN_HIP(ctx, hipMalloc((void**)&pack, skn_delta_pack_floats(st, n) * sizeof(float)));
    const int rc = skn_delta_rows(ctx, st, seq, r_dev, k_dev, v_dev, w_dev, a_dev, st->heads * st->dim, n, pack, out_dev);
    (void)hipStreamSynchronize(ctx->stream);
    (void)hipFree(pack);
    return rc;
}

}  // extern "C"
