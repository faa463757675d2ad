// Batched product of activations [m, k] with a stacked dense matrix [rows, k], both bf16 (v_mfma_f32_32x32x16_bf16) or
// both fp32 (v_mfma_f32_32x32x2_f32: true 32-bit products and sums), fp32 accumulation, epilogue in the store.
//
// Workgroup of WM x WN wavefronts, each with a tile of 32 TM tokens x 32 TN weight rows, walked along k in slices of 128
// bytes.  Both operands of a slice go from memory straight into LDS (16 bytes per lane, eight rows per request); the lane that
// fills slot s of row r fetches piece s ^ ((r / 2) % 8) of the row, so that the fragment reads -- the same piece of 32
// consecutive rows -- touch all 64 banks per sixteen lanes.  ST slices are in LDS at once: one bare barrier per slice, which
// says both "everyone's requests for this slice have landed" and "everyone is done with the slice before it", whose
// buffer the next request may overwrite.  Within a slice the fragments of a k-step are read while the products of the one
// before it run.
// The weights are the row operand, so that a lane's accumulators are runs of four consecutive outputs of one token.
// The fp32 form reads the same 16-byte pieces (four elements, half a wavefront each) and issues four matrix instructions
// per piece: k is summed in another order than it lies in memory, the same for both operands.
#include "dense.h"

#include <type_traits>

namespace {

typedef short bf16x8_t __attribute__((ext_vector_type(8)));
typedef __bf16 bf16x8_v __attribute__((ext_vector_type(8)));
typedef uint32_t u32x4 __attribute__((ext_vector_type(4)));
typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef float float16_t __attribute__((ext_vector_type(16)));

constexpr int kSlice = 128;  // bytes of k per slice

// KG groups of WM x WN wavefronts share the slices of a tile in turn; their sums meet in the epilogue.
template <int WM_, int WN_, int TM_, int TN_, int ST_, int KG_ = 1>
struct Shape {
    static constexpr int WM = WM_, WN = WN_, TM = TM_, TN = TN_, ST = ST_, KG = KG_;
    static constexpr int kThreads = 64 * WM * WN * KG, kRowsA = 32 * TM * WM, kRowsW = 32 * TN * WN;
    static constexpr int kBuf = (kRowsA + kRowsW) * kSlice;
    // the epilogue passes 32 WM tokens of the tile at a time through LDS
    static constexpr int kPitch = kRowsW + 4, kOutBytes = 32 * WM * kPitch * 4;
    static constexpr int kLds = KG * (ST * kBuf > kOutBytes ? ST * kBuf : kOutBytes);
};

__device__ __forceinline__ uint32_t half_bits(float f) { return __half_as_ushort(__float2half_rn(f)); }

template <typename T>
__device__ __forceinline__ float16_t mma(const u32x4& a, const u32x4& b, float16_t c) {
    if constexpr (std::is_same<T, float>::value) {
        const f32x4 x = __builtin_bit_cast(f32x4, a), y = __builtin_bit_cast(f32x4, b);
        c = __builtin_amdgcn_mfma_f32_32x32x2f32(x.x, y.x, c, 0, 0, 0);
        c = __builtin_amdgcn_mfma_f32_32x32x2f32(x.y, y.y, c, 0, 0, 0);
        c = __builtin_amdgcn_mfma_f32_32x32x2f32(x.z, y.z, c, 0, 0, 0);
        return __builtin_amdgcn_mfma_f32_32x32x2f32(x.w, y.w, c, 0, 0, 0);
    } else {
        return __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8_v, a), __builtin_bit_cast(bf16x8_v, b), c, 0, 0, 0);
    }
}

// T: uint16_t (bf16) or float.  lda_b, ldw_b: row pitches in bytes; slices = k_pad bytes / 128.
template <typename T, typename S>
__global__ __launch_bounds__(S::kThreads) void dense_gemm_kernel(const uint8_t* __restrict__ a, int64_t lda_b, int m, const uint8_t* __restrict__ w,
                                                                 int64_t ldw_b, int rows, int slices, int tiles_m, int tiles,
                                                                 const float* __restrict__ bias, const skn_dense_out out) {
    extern __shared__ __align__(16) uint8_t lds[];
    constexpr int WM = S::WM, WN = S::WN, TM = S::TM, TN = S::TN, ST = S::ST, KG = S::KG, kRowsA = S::kRowsA, kRowsW = S::kRowsW;
    constexpr int kReq = (kRowsA + kRowsW) / 8 / (WM * WN);  // requests per wavefront and slice
    const int tid = threadIdx.x, lane = tid & 63;
    const int all_wave = __builtin_amdgcn_readfirstlane(tid >> 6), group = all_wave / (WM * WN), wave = all_wave % (WM * WN);
    // An XCD (blockIdx % 8) takes consecutive tiles, which run down up to eight token tiles before they move on to the next
    // weight tile: what is resident on an XCD at a time shares both operands in its L2.
    const int per = (tiles + 7) / 8, tile = (int)(blockIdx.x & 7) * per + (int)(blockIdx.x >> 3);
    if (tile >= tiles || (int)(blockIdx.x >> 3) >= per) return;
    const int tiles_n = tiles / tiles_m, band = tile / (8 * tiles_n), band_m = min(8, tiles_m - 8 * band), in_band = tile - band * 8 * tiles_n;
    const int m0 = (8 * band + in_band % band_m) * kRowsA, n0 = in_band / band_m * kRowsW;

    const uint8_t* src[kReq];
    int dst[kReq];
#pragma unroll
    for (int i = 0; i < kReq; i++) {
        const int block = wave * kReq + i, r = block * 8 + (lane >> 3);  // row of the stacked A | W buffer
        const int piece = (lane & 7) ^ ((r >> 1) & 7);
        src[i] = (block * 8 < kRowsA ? a + (int64_t)min(m0 + r, m - 1) * lda_b
                                     : w + (int64_t)min(n0 + r - kRowsA, rows - 1) * ldw_b) + piece * 16;
        dst[i] = block * 1024;
    }
    // the group's i-th slice is slice KG i + group of the tile
    const int own = (slices - group + KG - 1) / KG, turns = (slices + KG - 1) / KG;
    auto request = [&](int i_own) __attribute__((always_inline)) {
        const int buf = (group * ST + i_own % ST) * S::kBuf, slice = KG * i_own + group;
#pragma unroll
        for (int i = 0; i < kReq; i++)
            __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void*)(src[i] + (int64_t)slice * kSlice),
                                             (__attribute__((address_space(3))) void*)(lds + buf + dst[i]), 16, 0, 0);
    };

    float16_t acc[TN][TM];
#pragma unroll
    for (int i = 0; i < TN; i++)
#pragma unroll
        for (int j = 0; j < TM; j++)
#pragma unroll
            for (int x = 0; x < 16; x++) acc[i][j][x] = 0.f;

    const int wv_m = wave % WM, wv_n = wave / WM, wm = wv_m * 32 * TM, wn = wv_n * 32 * TN, h = lane >> 5, r32 = lane & 31;
    const uint8_t* frag_a = lds + (wm + r32) * kSlice;
    const uint8_t* frag_w = lds + (kRowsA + wn + r32) * kSlice;
    const int swz = (r32 >> 1) & 7;  // (the 32-row blocks start at multiples of 16 rows: the same for all of them)

#pragma unroll
    for (int s = 0; s < ST - 1; s++)
        if (s < own) request(s);
    for (int s = 0; s < turns; s++) {
        // requests complete in order: all but the newest ST - 2 slices' have landed (near the end there are fewer newer ones: all)
        if (s + ST - 2 < own) asm volatile("s_waitcnt vmcnt(%0)" ::"n"(kReq * (ST - 2)) : "memory");
        else asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");
        if (s + ST - 1 < own) request(s + ST - 1);
        if (KG > 1 && s >= own) continue;
        const int buf = (group * ST + s % ST) * S::kBuf;
        u32x4 fa[2][TM], fw[2][TN];
        auto read = [&](int step) __attribute__((always_inline)) {
            const int off = buf + (((2 * step + h) ^ swz) * 16);
#pragma unroll
            for (int j = 0; j < TM; j++) fa[step & 1][j] = *reinterpret_cast<const u32x4*>(frag_a + off + j * 32 * kSlice);
#pragma unroll
            for (int i = 0; i < TN; i++) fw[step & 1][i] = *reinterpret_cast<const u32x4*>(frag_w + off + i * 32 * kSlice);
        };
        read(0);
#pragma unroll
        for (int step = 0; step < 4; step++) {
            if (step < 3) read(step + 1);
            __builtin_amdgcn_sched_barrier(0);
#pragma unroll
            for (int i = 0; i < TN; i++)
#pragma unroll
                for (int j = 0; j < TM; j++) acc[i][j] = mma<T>(fw[step & 1][i], fa[step & 1][j], acc[i][j]);
            __builtin_amdgcn_sched_barrier(0);
        }
    }

    // The tile goes through LDS (register x of lane 32 h + n: output row 8 (x / 4) + 4 h + x % 4 of its block, token n), so
    // that the epilogue is one short loop in which a thread has four consecutive outputs of one token and the threads
    // of a wavefront store whole rows of the tile.
    constexpr int kPitch = S::kPitch, kQuads = kRowsW / 4;
    float* tile_c = reinterpret_cast<float*>(lds);
    constexpr int kPart = 32 * WM * kPitch;  // floats of a group's pass
    const int q4 = 4 * (tid % kQuads), row = n0 + q4;  // (this thread's four rows are the same in every turn)
    int si = -1;
    for (int q = 0; q < out.nseg; q++)
        if (row >= out.seg[q].row0) si = q;
    const skn_dense_seg sg = out.seg[si < 0 ? 0 : si];
    // rows of the segment from here on
    const int left = row >= rows || (out.nseg && si < 0) ? 0 : out.nseg ? sg.row0 + sg.rows - row : out.resid_rows - row;
    const float4 b = bias && left > 0 ? *reinterpret_cast<const float4*>(bias + row) : make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
    for (int j = 0; j < TM; j++) {
        __syncthreads();  // (the fragments, then the pass before this one, have been read)
#pragma unroll
        for (int i = 0; i < TN; i++)
#pragma unroll
            for (int g = 0; g < 4; g++)
                *reinterpret_cast<float4*>(tile_c + group * kPart + (32 * wv_m + r32) * kPitch + wn + 32 * i + 8 * g + 4 * h) =
                    make_float4(acc[i][j][4 * g], acc[i][j][4 * g + 1], acc[i][j][4 * g + 2], acc[i][j][4 * g + 3]);
        __syncthreads();
        if (left <= 0) continue;
        for (int tl = tid / kQuads; tl < 32 * WM; tl += S::kThreads / kQuads) {
            const int t = m0 + (tl >> 5) * 32 * TM + 32 * j + (tl & 31);
            if (t >= m) continue;
            float4 c = *reinterpret_cast<const float4*>(tile_c + tl * kPitch + q4);
#pragma unroll
            for (int k = 1; k < KG; k++) {
                const float4 d = *reinterpret_cast<const float4*>(tile_c + k * kPart + tl * kPitch + q4);
                c = make_float4(c.x + d.x, c.y + d.y, c.z + d.z, c.w + d.w);
            }
            float v[4] = {c.x + b.x, c.y + b.y, c.z + b.z, c.w + b.w};
            if (out.nseg == 0) {
                float* p = out.resid + (int64_t)t * out.ldr + row;
                if (left >= 4) {
                    const float4 x = *reinterpret_cast<const float4*>(p);
                    *reinterpret_cast<float4*>(p) = make_float4(fmaf(out.mult, v[0], x.x), fmaf(out.mult, v[1], x.y), fmaf(out.mult, v[2], x.z),
                                                                fmaf(out.mult, v[3], x.w));
                } else {
                    for (int e = 0; e < left; e++) p[e] = fmaf(out.mult, e == 0 ? v[0] : e == 1 ? v[1] : v[2], p[e]);
                }
                continue;
            }
#pragma unroll
            for (int e = 0; e < 4; e++) v[e] = skn_dense_op(sg.op, v[e], sg.p0, sg.p1);
            if (si == out.mul_seg) {
                const int64_t from = (int64_t)out.mul_tokens[t] * out.mul_ld + out.mul_col + (row - sg.row0);
#pragma unroll
                for (int e = 0; e < 4; e++) v[e] *= e < left ? skn_table_at(out.mul_table, out.mul_type, from + e) : 0.f;
            }
            const int64_t at = (int64_t)t * sg.ldo + (row - sg.row0);
            if (left >= 4 && sg.out_type == SKN_TYPE_F32) {
                *reinterpret_cast<float4*>((float*)sg.out + at) = make_float4(v[0], v[1], v[2], v[3]);
            } else if (left >= 4) {
                if (sg.out_type == SKN_TYPE_F16)
                    *reinterpret_cast<uint2*>((uint16_t*)sg.out + at) = make_uint2(half_bits(v[0]) | (half_bits(v[1]) << 16), half_bits(v[2]) | (half_bits(v[3]) << 16));
                else *reinterpret_cast<uint2*>((uint16_t*)sg.out + at) = make_uint2(skn_bf16_bits(v[0]) | ((uint32_t)skn_bf16_bits(v[1]) << 16),
                                                                                skn_bf16_bits(v[2]) | ((uint32_t)skn_bf16_bits(v[3]) << 16));
            } else {
                for (int e = 0; e < left; e++) {
                    const float f = e == 0 ? v[0] : e == 1 ? v[1] : v[2];
                    if (sg.out_type == SKN_TYPE_F32) ((float*)sg.out)[at + e] = f;
                    else ((uint16_t*)sg.out)[at + e] = sg.out_type == SKN_TYPE_F16 ? (uint16_t)half_bits(f) : skn_bf16_bits(f);
                }
            }
        }
    }
}

using Tile64x64 = Shape<2, 2, 1, 1, 3>;
using Tile32x64Split = Shape<1, 2, 1, 1, 3, 4>;  // for few outputs: more and shorter chains of slices
using Tile128x64 = Shape<2, 2, 2, 1, 3>;
using Tile128x128 = Shape<2, 2, 2, 2, 2>;
using Tile256x256 = Shape<4, 2, 2, 4, 2>;

template <typename T, typename S>
int launch_gemm(skn_ctx* ctx, const skn_dense_mat& w, const void* a, int lda, int m, const skn_dense_out& out) {
    const int tm = (m + S::kRowsA - 1) / S::kRowsA, tn = (w.rows + S::kRowsW - 1) / S::kRowsW, tiles = tm * tn;
    skn_launch(ctx, dense_gemm_kernel<T, S>, dim3((unsigned)((tiles + 7) / 8 * 8)), dim3(S::kThreads), (size_t)S::kLds, (const uint8_t*)a,
               (int64_t)lda * (int64_t)sizeof(T), m, (const uint8_t*)w.w, (int64_t)w.k_pad * (int64_t)sizeof(T), w.rows,
               (int)(w.k_pad * sizeof(T) / kSlice), tm, tiles, w.bias, out);
    SKN_LAUNCH_CHECK(ctx);
    return SKN_OK;
}

template <typename T>
int pick_gemm(skn_ctx* ctx, const skn_dense_mat& w, const void* a, int lda, int m, const skn_dense_out& out) {
    // Each shape's time for one tile per compute unit and for as many as are resident, in relative units measured at k = 4096
    // (the larger the tile, the less it moves per product; the smaller, the fewer compute units wait at the end).
    struct Cost {
        int rows_a, rows_w, resident;
        float alone, full;
    };
    const Cost costs[4] = {{64, 64, 3, 25.f, 40.f}, {128, 64, 2, 31.f, 48.f}, {128, 128, 2, 59.f, 87.f}, {256, 256, 1, 145.f, 145.f}};
    int best = 0;
    float best_time = INFINITY;
    for (int i = 0; i < 4; i++) {
        const Cost& c = costs[i];
        const int tiles = ((m + c.rows_a - 1) / c.rows_a) * ((w.rows + c.rows_w - 1) / c.rows_w), round = c.resident * ctx->compute_units;
        const int rest = tiles % round;
        const float time = tiles / round * c.full + (rest == 0 ? 0.f : rest <= ctx->compute_units ? c.alone : c.full);
        if (time < best_time) best = i, best_time = time;
    }
    if (((m + 31) / 32) * ((w.rows + 63) / 64) <= ctx->compute_units && w.k_pad * (int)sizeof(T) >= 16 * kSlice) best = 4;
    if (ctx->opt_dense_tile > 0) best = ctx->opt_dense_tile - 1;
    switch (best) {
        case 0: return launch_gemm<T, Tile64x64>(ctx, w, a, lda, m, out);
        case 1: return launch_gemm<T, Tile128x64>(ctx, w, a, lda, m, out);
        case 2: return launch_gemm<T, Tile128x128>(ctx, w, a, lda, m, out);
        case 4: return launch_gemm<T, Tile32x64Split>(ctx, w, a, lda, m, out);
        default: return launch_gemm<T, Tile256x256>(ctx, w, a, lda, m, out);
    }
}

template <typename T, typename S>
int allow_lds(skn_ctx* ctx) {
    SKN_HIP(ctx, hipFuncSetAttribute((const void*)dense_gemm_kernel<T, S>, hipFuncAttributeMaxDynamicSharedMemorySize, S::kLds));
    return SKN_OK;
}

template <typename T>
int allow_all(skn_ctx* ctx) {
    SKN_TRY((allow_lds<T, Tile64x64>(ctx)));
    SKN_TRY((allow_lds<T, Tile32x64Split>(ctx)));
    SKN_TRY((allow_lds<T, Tile128x64>(ctx)));
    SKN_TRY((allow_lds<T, Tile128x128>(ctx)));
    return allow_lds<T, Tile256x256>(ctx);
}

int dense_gemm_init(skn_ctx* ctx) {
    SKN_TRY(allow_all<uint16_t>(ctx));
    return allow_all<float>(ctx);
}
skn_family register_family(dense_gemm_init);

}  // namespace

int skn_dense_gemm(skn_ctx* ctx, const skn_dense_mat& w, const void* a, int lda, int m, const skn_dense_out& out) {
    SKN_REQUIRE(ctx, w.w && a && m > 0 && w.rows > 0 && w.rows % kDenseRowPad == 0 && w.k_pad > 0 && w.k_pad % kDenseColPad == 0, SKN_ERR_ARG,
                "dense GEMM: bad shape (%d tokens, %d x %d)", m, w.rows, w.k_pad);
    SKN_REQUIRE(ctx, lda >= w.k_pad && lda % kDenseColPad == 0, SKN_ERR_SHAPE, "dense GEMM: activation pitch %d for %d columns", lda, w.k_pad);
    SKN_REQUIRE(ctx, (((uintptr_t)w.w | (uintptr_t)a) & 15) == 0, SKN_ERR_ARG, "dense GEMM: operands must be 16-byte aligned");
    SKN_REQUIRE(ctx, out.nseg >= 0 && out.nseg <= kDenseMaxSegs && (out.nseg > 0 || out.resid), SKN_ERR_ARG, "dense GEMM: no output");
    for (int i = 0; i < out.nseg; i++)
        SKN_REQUIRE(ctx, out.seg[i].out && out.seg[i].row0 % kDenseRowPad == 0 && out.seg[i].ldo % 4 == 0 && ((uintptr_t)out.seg[i].out & 15) == 0 &&
                             out.seg[i].row0 + skn_pad_rows(out.seg[i].rows) <= w.rows && (i == 0 || out.seg[i].row0 > out.seg[i - 1].row0),
                    SKN_ERR_ARG, "dense GEMM: segment %d is misplaced", i);
    SKN_REQUIRE(ctx, out.mul_seg < 0 || (out.mul_table && out.mul_tokens), SKN_ERR_ARG, "dense GEMM: no table to multiply with");
    SKN_REQUIRE(ctx, out.nseg > 0 || (out.ldr % 4 == 0 && out.resid_rows <= w.rows && ((uintptr_t)out.resid & 15) == 0), SKN_ERR_ARG,
                "dense GEMM: bad residual rows");
    if (w.type == SKN_TYPE_BF16) return pick_gemm<uint16_t>(ctx, w, a, lda, m, out);
    if (w.type == SKN_TYPE_F32) return pick_gemm<float>(ctx, w, a, lda, m, out);
    return skn_fail(ctx, SKN_ERR_TYPE, "dense GEMM: weights of type %d (BF16 or F32)", w.type);
}
