// Gated delta rule with a decay per key channel, behind short causal convolutions (state: rstate.h).
//
//   S <- g_t S;   u_t = beta_t (v_t - S^T k_t);   S <- S + k_t u_t^T;   o_t = S^T q_t         (g_t scales the rows of S)
//
// Everything here is fp32, the matrix instructions (v_mfma_f32_16x16x4_f32) included.  On prompts sixteen tokens (a chunk) are one
// step of the chain, as in csrc/delta.hip.  With W(s, t) the product of the factors of tokens s .. t of the chunk and S the state
// before it,
//   (I + L) U = beta (V - K0 S),   L_ts = beta_t k_t^T W(s+1, t) k_s for s < t,   K0_t = k_t W(0, t)
//   O = R0 S + G U,                R0_t = q_t W(0, t),   G_ts = q_t^T W(s+1, t) k_s for s <= t
//   S' = W(0, 15) S + sum_s k_s W(s+1, 15) u_s
// gated_chunk_kernel -- one wavefront per chunk and head, all chunks at once -- leaves V1 = (I + L)^-1 beta V, -K1 = -(I + L)^-1
// beta K0, R0, G and the decayed keys as operands; gated_scan_kernel walks the chunks: U = V1 - K1 S, and so on.
// Factors may be as small as they like (a channel may forget everything in a token), so no product of them is ever divided by
// another: the pair (s, t) is taken at the level b = 8, 4, 2 or 1 at which it falls into the two halves of a block of 2 b tokens,
// where W(s+1, t) is the product of the factors from s + 1 to the end of the lower half and those of the upper half up to t -- both
// at most one, one on each operand.
#include "delta.h"
#include "dense.h"
#include "rstate.h"

#include <algorithm>

namespace {

constexpr int kTrash = 64;  // floats behind the operands that take the outputs of tokens past the end

__device__ __forceinline__ float silu(float z) { return z * skn_sigmoid(z); }
// log2 of a channel's factor
__device__ __forceinline__ float log2_factor(float z, float rate) {
    const float softplus = z > 15.f ? z + __expf(-z) : log1pf(__expf(z));
    return -1.4426950408889634f * rate * softplus;
}

// ---- convolutions ---------------------------------------------------------------------------------------------------------------

struct ConvArgs {
    const float *q, *k, *v;  // [n][ld], this portion's inputs
    int ld, n, pos0;
    const float* ring;  // inputs of the tokens before it
    const float* taps;  // [channels][n_taps]
    int n_taps, kv_heads, dim, vcols, channels;
    float *cq, *ck, *cv;
};

constexpr int kMaxTaps = 8, kConvRows = 8;

// rows t0 .. t0 + 7 of channel c (of the ring and the taps), whose inputs in the portion are src[row * ld]; past the end: the last row
__device__ __forceinline__ void conv_rows(const ConvArgs& a, const float* src, int c, int t0, float (&y)[kConvRows]) {
    float w[kMaxTaps], x[kConvRows + kMaxTaps - 1];  // w[j]: of the input j tokens back; x[i]: of row t0 - 7 + i
#pragma unroll
    for (int j = 0; j < kMaxTaps; j++) w[j] = j < a.n_taps ? a.taps[(int64_t)c * a.n_taps + a.n_taps - 1 - j] : 0.f;
#pragma unroll
    for (int i = 0; i < kConvRows + kMaxTaps - 1; i++) {
        const int t = t0 - (kMaxTaps - 1) + i, p = a.pos0 + t;
        x[i] = 0.f;
        if (i >= kMaxTaps - a.n_taps) {
            if (t >= 0) x[i] = src[(int64_t)min(t, a.n - 1) * a.ld];
            else if (p >= 0) x[i] = a.ring[(int64_t)(p % a.n_taps) * a.channels + c];
        }
    }
#pragma unroll
    for (int r = 0; r < kConvRows; r++) {
        float s = 0.f;
#pragma unroll
        for (int j = 0; j < kMaxTaps; j++) s = fmaf(x[r + kMaxTaps - 1 - j], w[j], s);
        y[r] = silu(s);
    }
}

// grid (rows / 8, units / 4): a wavefront takes the q or the k of a q/k head, or 64 value channels
__global__ __launch_bounds__(256) void conv_rows_kernel(const ConvArgs a) {
    const int t0 = blockIdx.x * kConvRows, unit = blockIdx.y * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63, qk = a.kv_heads * a.dim;
    const int rows = min(kConvRows, a.n - t0);
    float y[4][kConvRows];
    if (unit < 2 * a.kv_heads) {
        const int which = unit & 1, head = unit >> 1;
        const float* src = (which ? a.k : a.q) + head * a.dim;
        float* dst = (which ? a.ck : a.cq) + (int64_t)t0 * a.ld + head * a.dim;
        float ss[kConvRows];
#pragma unroll
        for (int r = 0; r < kConvRows; r++) ss[r] = 0.f;
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const int d = lane + 64 * i;
            if (64 * i >= a.dim) break;
            conv_rows(a, src + min(d, a.dim - 1), which * qk + head * a.dim + min(d, a.dim - 1), t0, y[i]);
#pragma unroll
            for (int r = 0; r < kConvRows; r++) ss[r] = d < a.dim ? fmaf(y[i][r], y[i][r], ss[r]) : ss[r];
        }
#pragma unroll
        for (int r = 0; r < kConvRows; r++) {
            const float f = (which ? 1.0f : 1.0f / sqrtf((float)a.dim)) / sqrtf(wave_sum(ss[r]) + kUnitEps);
#pragma unroll
            for (int i = 0; i < 4; i++)
                if (lane + 64 * i < a.dim && r < rows) dst[(int64_t)r * a.ld + lane + 64 * i] = y[i][r] * f;
        }
        return;
    }
    const int c = (unit - 2 * a.kv_heads) * 64 + lane;
    if (c >= a.vcols) return;
    conv_rows(a, a.v + c, 2 * qk + c, t0, y[0]);
#pragma unroll
    for (int r = 0; r < kConvRows; r++)
        if (r < rows) a.cv[(int64_t)(t0 + r) * a.ld + c] = y[0][r];
}

// the last tokens' inputs to the ring (after every row has read what was there); grid (channels / 256, tokens kept)
__global__ __launch_bounds__(256) void conv_keep_kernel(const ConvArgs a, float* __restrict__ ring) {
    const int c = blockIdx.x * 256 + threadIdx.x, t = a.n - 1 - (int)blockIdx.y, qk = a.kv_heads * a.dim;
    if (c >= a.channels) return;
    const float* src = c < qk ? a.q + c : c < 2 * qk ? a.k + (c - qk) : a.v + (c - 2 * qk);
    ring[(int64_t)((a.pos0 + t) % a.n_taps) * a.channels + c] = src[(int64_t)t * a.ld];
}

// ---- prompts --------------------------------------------------------------------------------------------------------------------

// Operands of a chunk and head, in floats from its start, in the layouts of csrc/delta.hip: -K1 and R0 as row operands (tiles of 16
// channels), the decayed keys by channel, G as a row operand, the factors of the whole chunk, V1 as a column operand.
__host__ __device__ constexpr int off_k1(int) { return 0; }
__host__ __device__ constexpr int off_r0(int dp) { return 16 * dp; }
__host__ __device__ constexpr int off_kt(int dp) { return 32 * dp; }
__host__ __device__ constexpr int off_g(int dp) { return 48 * dp; }
__host__ __device__ constexpr int off_w(int dp) { return 48 * dp + 256; }
__host__ __device__ constexpr int off_v(int dp) { return 49 * dp + 256; }
__host__ __device__ constexpr int chunk_floats(int dp, int vdim) { return off_v(dp) + 16 * ((vdim + 15) / 16 * 16); }

struct ChunkArgs {
    const float *q, *k, *v, *beta, *z;  // convolved q, k, v; [n][ld]
    const float* rate;                  // [heads]
    int ld, n, heads, per_kv, dim, vdim;
    float* ops;
};

template <int B>
__device__ __forceinline__ void level_factors(const float (&gl)[kChunk], float (&f)[kChunk]) {
#pragma unroll
    for (int block = 0; block < kChunk; block += 2 * B) {
        float acc = 0.f;
#pragma unroll
        for (int t = block + B; t < block + 2 * B; t++) acc += gl[t], f[t] = __builtin_amdgcn_exp2f(acc);
        acc = 0.f;
#pragma unroll
        for (int s = block + B - 1; s >= block; s--) f[s] = __builtin_amdgcn_exp2f(acc), acc += gl[s];
    }
}

// one wavefront per (chunk, head); tokens past n change nothing (q = k = v = beta = 0, factor 1)
template <int DP>
__global__ __launch_bounds__(64) void gated_chunk_kernel(const ChunkArgs p) {
    constexpr int kPitch = DP + 4, kSets = (DP + 63) / 64, kTiles = DP / 16;
    __shared__ __align__(16) float op[2][kChunk * kPitch];  // a level's q and k; then K0 and R0
    __shared__ __align__(16) float tri[2][kChunk][20];      // L, G
    const int lane = threadIdx.x, chunk = blockIdx.x, h = blockIdx.y, t0 = chunk * kChunk, t16 = lane & 15, q4 = lane >> 4;
    const int kvh = h / p.per_kv, dim = p.dim, last = p.n - 1;
    float* out = p.ops + ((int64_t)h * gridDim.x + chunk) * chunk_floats(DP, p.vdim);
    const float rate = p.rate[h];
    float beta[kChunk], q[kSets][kChunk], k[kSets][kChunk], gl[kSets][kChunk];  // this lane's channels; gl: log2 of the factors
#pragma unroll
    for (int t = 0; t < kChunk; t++) beta[t] = t0 + t < p.n ? p.beta[(int64_t)min(t0 + t, last) * p.ld + h] : 0.f;
#pragma unroll
    for (int i = 0; i < kSets; i++) {
        const int d = lane + 64 * i, dd = min(d, dim - 1);
#pragma unroll
        for (int t = 0; t < kChunk; t++) {
            const int64_t row = (int64_t)min(t0 + t, last) * p.ld;
            q[i][t] = p.q[row + kvh * dim + dd];
            k[i][t] = p.k[row + kvh * dim + dd];
            gl[i][t] = p.z[row + h * dim + dd];
        }
#pragma unroll
        for (int t = 0; t < kChunk; t++) {
            const bool in = d < dim && t0 + t < p.n;
            q[i][t] = in ? q[i][t] : 0.f;
            k[i][t] = in ? k[i][t] : 0.f;
            gl[i][t] = in ? log2_factor(gl[i][t], rate) : 0.f;
        }
    }
    // the triangles, level by level; level 0: the diagonal of G
    f32x4 kk = {0.f, 0.f, 0.f, 0.f}, qk = kk;
    auto level = [&](auto width) __attribute__((always_inline)) {
        constexpr int B = decltype(width)::value;
        __syncthreads();
#pragma unroll
        for (int i = 0; i < kSets; i++) {
            const int d = lane + 64 * i;
            if (d >= DP) continue;
            float f[kChunk];
#pragma unroll
            for (int t = 0; t < kChunk; t++) f[t] = 1.f;
            if constexpr (B > 0) level_factors<B>(gl[i], f);
#pragma unroll
            for (int t = 0; t < kChunk; t++) {
                op[0][t * kPitch + d] = q[i][t] * f[t];
                op[1][t * kPitch + d] = k[i][t] * f[t];
            }
        }
        __syncthreads();
        f32x4 x[2], y[2];
#pragma unroll
        for (int i = 0; i < 2; i++) x[i] = y[i] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 2
        for (int c = 0; c < kTiles; c++) {
            const int at = t16 * kPitch + 16 * c + 4 * q4;
            const f32x4 qv = load4(&op[0][at]), kv = load4(&op[1][at]);
#pragma unroll
            for (int e = 0; e < 4; e++) {
                if constexpr (B > 0) x[e & 1] = mma(kv[e], kv[e], x[e & 1]);
                y[e & 1] = mma(qv[e], kv[e], y[e & 1]);
            }
        }
#pragma unroll
        for (int e = 0; e < 4; e++) {
            const int t = 4 * q4 + e, s = t16, diff = t ^ s;
            const bool mine = B == 0 ? diff == 0 : t > s && diff >= B && diff < 2 * B;
            kk[e] = mine ? x[0][e] + x[1][e] : kk[e];
            qk[e] = mine ? y[0][e] + y[1][e] : qk[e];
        }
    };
    level(std::integral_constant<int, 0>());
    level(std::integral_constant<int, 8>());
    level(std::integral_constant<int, 4>());
    level(std::integral_constant<int, 2>());
    level(std::integral_constant<int, 1>());
#pragma unroll
    for (int e = 0; e < 4; e++) {
        const int t = 4 * q4 + e, s = t16;
        tri[0][t][s] = s < t ? kk[e] : 0.f;
        tri[1][t][s] = s <= t ? qk[e] : 0.f;
    }
    __syncthreads();
    // x_t = beta_t (rhs_t - sum_{s < t} (k_t W k_s) x_s)
    auto solve = [&](float (&x)[kChunk]) __attribute__((always_inline)) {
#pragma unroll
        for (int t = 0; t < kChunk; t++) {
#pragma unroll
            for (int s = 0; s < t; s++) x[t] = fmaf(-tri[0][t][s], x[s], x[t]);
            x[t] *= beta[t];
        }
    };
#pragma unroll
    for (int i = 0; i < kSets; i++) {
        const int d = lane + 64 * i;
        if (d >= DP) continue;
        float x[kChunk], upto = 0.f;
#pragma unroll
        for (int t = 0; t < kChunk; t++) {
            upto += gl[i][t];
            const float f = __builtin_amdgcn_exp2f(upto);
            x[t] = k[i][t] * f;
            op[1][t * kPitch + d] = q[i][t] * f;
        }
        out[off_w(DP) + d] = __builtin_amdgcn_exp2f(upto);
        solve(x);
#pragma unroll
        for (int t = 0; t < kChunk; t++) op[0][t * kPitch + d] = -x[t];
        float after = 0.f;
#pragma unroll
        for (int t = kChunk - 1; t >= 0; t--) {
            x[t] = k[i][t] * __builtin_amdgcn_exp2f(after);
            after += gl[i][t];
        }
        float* frag = out + off_kt(DP) + ((d >> 4) * 64 + (d & 15)) * 4;  // tile d / 16, lane 16 q + d % 16
#pragma unroll
        for (int q = 0; q < 4; q++) *reinterpret_cast<f32x4*>(frag + 64 * q) = f32x4{x[4 * q], x[4 * q + 1], x[4 * q + 2], x[4 * q + 3]};
    }
    for (int d = lane; d < (p.vdim + 15) / 16 * 16; d += 64) {
        float x[kChunk];
#pragma unroll
        for (int t = 0; t < kChunk; t++)
            x[t] = d < p.vdim && t0 + t < p.n ? p.v[(int64_t)min(t0 + t, last) * p.ld + h * p.vdim + min(d, p.vdim - 1)] : 0.f;
        solve(x);
        float* frag = out + off_v(DP) + ((d >> 4) * 64 + (d & 15)) * 4;
#pragma unroll
        for (int q = 0; q < 4; q++) *reinterpret_cast<f32x4*>(frag + 64 * q) = f32x4{x[4 * q], x[4 * q + 1], x[4 * q + 2], x[4 * q + 3]};
    }
    __syncthreads();
#pragma unroll 2
    for (int c = 0; c < kTiles; c++) {
        *reinterpret_cast<f32x4*>(out + off_k1(DP) + (c * 64 + lane) * 4) = load4(&op[0][t16 * kPitch + 16 * c + 4 * q4]);
        *reinterpret_cast<f32x4*>(out + off_r0(DP) + (c * 64 + lane) * 4) = load4(&op[1][t16 * kPitch + 16 * c + 4 * q4]);
    }
    *reinterpret_cast<f32x4*>(out + off_g(DP) + lane * 4) = load4(&tri[1][t16][4 * q4]);
}

template <int DP>
struct GatedOps {
    static constexpr int kTiles = DP / 16;
    f32x4 k1[kTiles], r0[kTiles], kt[kTiles], w[kTiles], v, g;
    __device__ __forceinline__ void load(const float* p, int lane, int tile) {
        v = load4(p + off_v(DP) + (tile * 64 + lane) * 4);
#pragma unroll
        for (int j = 0; j < kTiles; j++) {
            k1[j] = load4(p + off_k1(DP) + (j * 64 + lane) * 4);
            r0[j] = load4(p + off_r0(DP) + (j * 64 + lane) * 4);
        }
        g = load4(p + off_g(DP) + lane * 4);
#pragma unroll
        for (int j = 0; j < kTiles; j++) {
            kt[j] = load4(p + off_kt(DP) + (j * 64 + lane) * 4);
            w[j] = load4(p + off_w(DP) + 16 * j + 4 * (lane >> 4));
        }
    }
};

// One wavefront per head and tile of sixteen value columns, its part of S in accumulator layout (also the layout of a column operand);
// the wavefronts of a head are on one XCD (blockIdx % 8), as in delta_scan_kernel.
template <int DP>
__global__ __launch_bounds__(64) void gated_scan_kernel(const float* __restrict__ ops, int n, int chunks, int heads, int vdim, float* __restrict__ state,
                                                        float* __restrict__ o, float* __restrict__ trash) {
    constexpr int kTiles = DP / 16;
    const int lane = threadIdx.x, tiles = (vdim + 15) / 16, turn = (int)(blockIdx.x >> 3), h = (int)(blockIdx.x & 7) + 8 * (turn / tiles), tile = turn % tiles;
    if (h >= heads) return;
    const int col = 16 * tile + (lane & 15), size = chunk_floats(DP, vdim);
    const bool live = col < vdim;  // (lanes beyond the last column compute along and store nothing)
    float* sp = state + ((int64_t)h * vdim + min(col, vdim - 1)) * DP + 4 * (lane >> 4);
    f32x4 s[kTiles];
#pragma unroll
    for (int j = 0; j < kTiles; j++) s[j] = load4(sp + 16 * j);
    const float* src = ops + (int64_t)h * chunks * size;

    auto step = [&](const GatedOps<DP>& x, int chunk) __attribute__((always_inline)) {
        const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
        f32x4 u[2] = {x.v, zero}, z[2] = {zero, zero};
#pragma unroll
        for (int j = 0; j < kTiles; j++)
#pragma unroll
            for (int e = 0; e < 4; e++) {
                u[e & 1] = mma(x.k1[j][e], s[j][e], u[e & 1]);
                z[e & 1] = mma(x.r0[j][e], s[j][e], z[e & 1]);
            }
        u[0] += u[1];
#pragma unroll
        for (int j = 0; j < kTiles; j++) s[j] *= x.w[j];
#pragma unroll
        for (int e = 0; e < 4; e++) {
#pragma unroll
            for (int j = 0; j < kTiles; j++) s[j] = mma(x.kt[j][e], u[0][e], s[j]);
            z[e & 1] = mma(x.g[e], u[0][e], z[e & 1]);
        }
        z[0] += z[1];
        // (one store per token whatever the lane, so that the number of requests outstanding is known)
#pragma unroll
        for (int e = 0; e < 4; e++) {
            const int t = chunk * kChunk + 4 * (lane >> 4) + e;
            float* dst = live && t < n ? o + ((int64_t)t * heads + h) * vdim + col : trash + lane;
            *dst = z[0][e];
        }
    };
    GatedOps<DP> even;
    if constexpr (DP <= 128) {
        GatedOps<DP> odd;
        even.load(src, lane, tile);
        for (int c = 0; c < chunks; c += 2) {
            odd.load(src + (int64_t)min(c + 1, chunks - 1) * size, lane, tile);
            __builtin_amdgcn_sched_barrier(0);
            step(even, c);
            if (c + 1 == chunks) break;
            even.load(src + (int64_t)min(c + 2, chunks - 1) * size, lane, tile);
            __builtin_amdgcn_sched_barrier(0);
            step(odd, c + 1);
        }
    } else {
        for (int c = 0; c < chunks; c++) {
            even.load(src + (int64_t)c * size, lane, tile);
            step(even, c);
        }
    }
    if (live) {
#pragma unroll
        for (int j = 0; j < kTiles; j++) *reinterpret_cast<f32x4*>(sp + 16 * j) = s[j];
    }
}

// ---- one token --------------------------------------------------------------------------------------------------------------------

struct StepArgs {
    skn_gated_step p;
    const float* taps;
    const float* rate;
    int n_taps, heads, kv_heads, dim, vdim, channels;
    float* ring;
    float* state;
};

// row . t over rank_pad columns (zeros of the row from its rank on), shared by eight lanes; the total in all of them
template <typename W>
__device__ __forceinline__ float low_rank_dot(const W* row, const float* t, int rank_pad, int l) {
    float z = 0.f;
#pragma unroll 2
    for (int i = 8 * l; i < rank_pad; i += 64) {
        float f[8];
        const float4 a = *reinterpret_cast<const float4*>(t + i), b = *reinterpret_cast<const float4*>(t + i + 4);
        if constexpr (sizeof(W) == 2) {
            const uint4 w = *reinterpret_cast<const uint4*>(row + i);
            const uint32_t u[4] = {w.x, w.y, w.z, w.w};
#pragma unroll
            for (int j = 0; j < 4; j++) f[2 * j] = __uint_as_float(u[j] << 16), f[2 * j + 1] = __uint_as_float(u[j] & 0xFFFF0000u);
        } else {
            const float4 c = *reinterpret_cast<const float4*>(row + i), d = *reinterpret_cast<const float4*>(row + i + 4);
            f[0] = c.x, f[1] = c.y, f[2] = c.z, f[3] = c.w, f[4] = d.x, f[5] = d.y, f[6] = d.z, f[7] = d.w;
        }
        z += ((f[0] * a.x + f[1] * a.y) + (f[2] * a.z + f[3] * a.w)) + ((f[4] * b.x + f[5] * b.y) + (f[6] * b.z + f[7] * b.w));
    }
    return lane_group_sum<8>(z);
}

// one workgroup of NW wavefronts per head
template <int L, int NW, typename W>
__global__ __launch_bounds__(64 * NW) void gated_step_kernel(const StepArgs a) {
    constexpr int DP = 8 * L, CW = 64 / L, kThreads = 64 * NW, kCols = NW * CW, kPasses = 256 / kCols;  // columns per wavefront, per pass
    __shared__ __align__(16) float vec[3][DP];  // q, k, factors
    __shared__ float sv[256], sg[256], so[256], red[NW];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, h = blockIdx.x, rl = lane & (L - 1), per_kv = a.heads / a.kv_heads, kvh = h / per_kv;
    const int dim = a.dim, vdim = a.vdim, qk = a.kv_heads * dim;
    const skn_gated_step& p = a.p;
    // the state first: it does not wait for anything
    Vec8 s[kPasses];
    float* sp = a.state + ((int64_t)h * vdim) * DP + 8 * rl;
#pragma unroll
    for (int i = 0; i < kPasses; i++)
        if (i * kCols < vdim) s[i].load(sp + (int64_t)min(i * kCols + wave * CW + lane / L, vdim - 1) * DP);
    const int pos = p.state[1];
    const float beta = p.beta[h];
    // factors of the key channels and gates of the value channels: eight lanes per row of the second matrices
    for (int r = tid >> 3; r < DP + vdim; r += kThreads / 8) {
        const int d = r - DP, l = tid & 7;
        if (r < DP) {
            const float z = low_rank_dot((const W*)p.w_a + (int64_t)(h * dim + min(r, dim - 1)) * p.rank_a_pad, p.a_low, p.rank_a_pad, l);
            if (l == 0) vec[2][r] = r < dim ? __builtin_amdgcn_exp2f(log2_factor(z + p.bias_a[h * dim + r], a.rate[h])) : 0.f;
        } else {
            const float z = low_rank_dot((const W*)p.w_g + (int64_t)(h * vdim + d) * p.rank_g_pad, p.g_low, p.rank_g_pad, l);
            if (l == 0) sg[d] = skn_sigmoid(z);
        }
    }
    // convolutions: channels q, k of the head's q/k head, then v
    for (int i = tid; i < 2 * DP + vdim; i += kThreads) {
        const int which = i < DP ? 0 : i < 2 * DP ? 1 : 2, d = i - which * DP;
        if (which < 2 && d >= dim) {
            vec[which][d] = 0.f;
            continue;
        }
        const int c = which < 2 ? which * qk + kvh * dim + d : 2 * qk + h * vdim + d;
        const float x = (which == 0 ? p.q + kvh * dim : which == 1 ? p.k + kvh * dim : p.v + h * vdim)[d];
        const float* w = a.taps + (int64_t)c * a.n_taps;
        float y = x * w[a.n_taps - 1];
        for (int j = 1; j < a.n_taps; j++) {
            const int at = pos - j;
            if (at >= 0) y = fmaf(a.ring[(int64_t)(at % a.n_taps) * a.channels + c], w[a.n_taps - 1 - j], y);
        }
        // (this token's slot is none of those that are read; the heads that share a q/k head leave it to the first)
        if (which == 2 || h % per_kv == 0) a.ring[(int64_t)(pos % a.n_taps) * a.channels + c] = x;
        if (which < 2) vec[which][d] = silu(y);
        else sv[d] = silu(y);
    }
    __syncthreads();
    float sq = 0.f, sk = 0.f;  // (every wavefront for itself)
    for (int d = lane; d < DP; d += 64) sq = fmaf(vec[0][d], vec[0][d], sq), sk = fmaf(vec[1][d], vec[1][d], sk);
    const float fq = 1.0f / (sqrtf(wave_sum(sq) + kUnitEps) * sqrtf((float)dim)), fk = 1.0f / sqrtf(wave_sum(sk) + kUnitEps);
    Vec8 q, k, g;
    q.load(&vec[0][8 * rl]);
    k.load(&vec[1][8 * rl]);
    g.load(&vec[2][8 * rl]);
#pragma unroll
    for (int j = 0; j < 8; j++) q.v[j] *= fq, k.v[j] *= fk;
#pragma unroll
    for (int i = 0; i < kPasses; i++) {
        if (i * kCols >= vdim) break;
        const int col = i * kCols + wave * CW + lane / L;
#pragma unroll
        for (int j = 0; j < 8; j++) s[i].v[j] *= g.v[j];
        const float u = beta * (sv[min(col, vdim - 1)] - dot_over_lanes<L>(k, s[i]));
#pragma unroll
        for (int j = 0; j < 8; j++) s[i].v[j] = fmaf(k.v[j], u, s[i].v[j]);
        const float o = dot_over_lanes<L>(q, s[i]);
        if (col < vdim) {
            s[i].store(sp + (int64_t)col * DP);
            if (rl == 0) so[col] = o;
        }
    }
    __syncthreads();
    float ss = 0.f;
    for (int d = tid; d < vdim; d += kThreads) ss = fmaf(so[d], so[d], ss);
    ss = wave_sum(ss);
    if (lane == 0) red[wave] = ss;
    __syncthreads();
    ss = 0.f;
#pragma unroll
    for (int i = 0; i < NW; i++) ss += red[i];
    const float inv = 1.0f / sqrtf(ss / (float)vdim + p.eps);
    for (int d = tid; d < vdim; d += kThreads) p.y[h * vdim + d] = so[d] * inv * p.norm[h * vdim + d] * sg[d];
}

template <int DP>
int launch_rows(skn_ctx* ctx, const skn_rstate* st, const ChunkArgs& a, float* state, float* o) {
    const int chunks = (a.n + kChunk - 1) / kChunk, tiles = (a.vdim + 15) / 16;
    skn_launch(ctx, gated_chunk_kernel<DP>, dim3(chunks, a.heads), dim3(64), 0, a);
    SKN_LAUNCH_CHECK(ctx);
    float* trash = a.ops + (size_t)chunks * a.heads * chunk_floats(DP, a.vdim);
    skn_launch(ctx, gated_scan_kernel<DP>, dim3((unsigned)((a.heads + 7) / 8 * 8 * tiles)), dim3(64), 0, (const float*)a.ops, a.n, chunks, a.heads, a.vdim, state, o,
               trash);
    SKN_LAUNCH_CHECK(ctx);
    return SKN_OK;
}

template <int L, int NW>
int launch_step(skn_ctx* ctx, const StepArgs& a) {
    if (a.p.w_type == SKN_TYPE_F32) skn_launch(ctx, gated_step_kernel<L, NW, float>, dim3(a.heads), dim3(64 * NW), 0, a);
    else skn_launch(ctx, gated_step_kernel<L, NW, uint16_t>, dim3(a.heads), dim3(64 * NW), 0, a);
    SKN_LAUNCH_CHECK(ctx);
    return SKN_OK;
}

}  // namespace

size_t skn_gated_delta_pack_floats(const skn_rstate* st, int n) {
    return (size_t)((n + kChunk - 1) / kChunk) * st->heads * chunk_floats(st->dim_pad, st->vdim) + kTrash;
}

int skn_gated_delta_rows(skn_ctx* ctx, skn_rstate* st, int seq, const skn_channel_delta& p, const float* q, const float* k, const float* v, const float* beta,
                         const float* z, int ld, int n, int pos0, float* cq, float* ck, float* cv, float* pack, float* o) {
    SKN_REQUIRE(ctx, st->taps > 0, SKN_ERR_STATE, "gated delta rule: the state has no convolutions");
    SKN_REQUIRE(ctx, n > 0 && st->heads <= 65535, SKN_ERR_SHAPE, "gated delta rule: %d tokens x %d heads", n, st->heads);
    ConvArgs c = {q, k, v, ld, n, pos0, st->seq_conv(seq), p.conv, st->taps, st->kv_heads, st->dim, st->heads * st->vdim, st->channels, cq, ck, cv};
    const int units = 2 * st->kv_heads + (c.vcols + 63) / 64;
    skn_launch(ctx, conv_rows_kernel, dim3((n + kConvRows - 1) / kConvRows, (units + 3) / 4), dim3(256), 0, c);
    SKN_LAUNCH_CHECK(ctx);
    skn_launch(ctx, conv_keep_kernel, dim3((st->channels + 255) / 256, std::min(n, st->taps)), dim3(256), 0, c, st->seq_conv(seq));
    SKN_LAUNCH_CHECK(ctx);
    const ChunkArgs a = {cq, ck, cv, beta, z, p.decay_rate, ld, n, st->heads, st->heads / st->kv_heads, st->dim, st->vdim, pack};
    float* s = st->seq_state(seq);
    switch (st->dim_pad) {
        case 32: return launch_rows<32>(ctx, st, a, s, o);
        case 64: return launch_rows<64>(ctx, st, a, s, o);
        case 128: return launch_rows<128>(ctx, st, a, s, o);
        default: return launch_rows<256>(ctx, st, a, s, o);
    }
}

int skn_gated_step_launch(skn_ctx* ctx, skn_rstate* st, int seq, const skn_channel_delta& c, const skn_gated_step& p) {
    SKN_REQUIRE(ctx, st->taps > 0, SKN_ERR_STATE, "gated delta rule: the state has no convolutions");
    const StepArgs a = {p, c.conv, c.decay_rate, st->taps, st->heads, st->kv_heads, st->dim, st->vdim, st->channels, st->seq_conv(seq), st->seq_state(seq)};
    switch (st->dim_pad) {
        case 32: return launch_step<4, 4>(ctx, a);
        case 64: return launch_step<8, 8>(ctx, a);
        case 128: return launch_step<16, 16>(ctx, a);
        default: return launch_step<32, 16>(ctx, a);
    }
}

extern "C" int skn_gated_delta(skn_ctx* ctx, skn_rstate* st, int seq, const skn_channel_delta* p, const float* q_dev, const float* k_dev, const float* v_dev,
                               const float* beta_dev, const float* z_dev, int n, float* out_dev) {
    SKN_REQUIRE(nullptr, ctx != nullptr, SKN_ERR_ARG, "skn_gated_delta: ctx is null");
    SKN_REQUIRE(ctx, st && p && p->conv && p->decay_rate && q_dev && k_dev && v_dev && beta_dev && z_dev && out_dev, SKN_ERR_ARG, "skn_gated_delta: null pointer");
    SKN_REQUIRE(ctx, seq >= 0 && seq < st->n_seq && n > 0, SKN_ERR_RANGE, "skn_gated_delta: %d tokens of sequence %d of %d", n, seq, st->n_seq);
    // (the rows' kernels take one pitch: the callers' tight rows are spread to it)
    const int qk = st->kv_heads * st->dim, vc = st->heads * st->vdim, zc = st->heads * st->dim, ld = std::max(qk, std::max(vc, zc));
    const size_t col = (size_t)n * ld;
    float* m = nullptr;
    SKN_HIP(ctx, hipMalloc((void**)&m, (8 * col + skn_gated_delta_pack_floats(st, n)) * sizeof(float)));
    const float* src[5] = {q_dev, k_dev, v_dev, beta_dev, z_dev};
    const int cols[5] = {qk, qk, vc, st->heads, zc};
    int rc = SKN_OK;
    for (int i = 0; i < 5 && rc == SKN_OK; i++)
        if (hipMemcpy2DAsync(m + i * col, (size_t)ld * 4, src[i], (size_t)cols[i] * 4, (size_t)cols[i] * 4, n, hipMemcpyDeviceToDevice, ctx->stream) != hipSuccess)
            rc = skn_fail(ctx, SKN_ERR_HIP, "skn_gated_delta: copy failed");
    if (rc == SKN_OK)
        rc = skn_gated_delta_rows(ctx, st, seq, *p, m, m + col, m + 2 * col, m + 3 * col, m + 4 * col, ld, n, st->pos[seq], m + 5 * col, m + 6 * col, m + 7 * col,
                                  m + 8 * col, out_dev);
    if (rc == SKN_OK) st->pos[seq] += n;
    (void)hipStreamSynchronize(ctx->stream);
    (void)hipFree(m);
    return rc;
}
