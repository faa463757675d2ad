// Batched product of activations [m, k] with a stacked dense matrix [rows, k], both bf16 (v_mfma_f32_32x32x16_bf16) or
// both fp32 (v_mfma_f32_32x32x2_f32: true 32-bit products and sums), fp32 accumulation, epilogue in the store.
//
// Workgroup of four wavefronts (2 x 2), tile (64 TM) tokens x (64 TN) weight rows, walked along k in slices of 128 bytes.
// Both tiles of a slice go from memory straight into LDS (16 bytes per lane, eight rows per request); the lane that
// fills slot s of row r fetches piece s ^ ((r / 2) % 8) of the row, so that the fragment reads -- the same piece of 32
// consecutive rows -- touch all 64 banks per sixteen lanes.  kStages slices are in flight: one bare barrier per slice, which
// says both "everyone's requests for this slice have landed" and "everyone is done with the slice before it", whose
// buffer the next request may overwrite.
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

constexpr int kStages = 3;
constexpr int kSlice = 128;  // bytes of k per slice

template <int TM, int TN>
constexpr int gemm_lds_bytes() {
    return kStages * 64 * (TM + TN) * kSlice;
}

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
template <typename T, int TM, int TN>
__global__ __launch_bounds__(256) void dense_gemm_kernel(const uint8_t* __restrict__ a, int64_t lda_b, int m, const uint8_t* __restrict__ w,
                                                         int64_t ldw_b, int rows, int slices, int tiles_m, int tiles,
                                                         const float* __restrict__ bias, const skn_dense_out out) {
    extern __shared__ __align__(16) uint8_t lds[];
    constexpr int kRowsA = 64 * TM, kRowsW = 64 * TN, kBuf = (kRowsA + kRowsW) * kSlice;
    constexpr int kReq = (kRowsA + kRowsW) / 8 / 4;  // requests per wavefront and slice
    const int tid = threadIdx.x, lane = tid & 63;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    // consecutive workgroups of an XCD (blockIdx % 8) share a weight tile: it comes from memory once per XCD
    const int per = (tiles + 7) / 8, tile = (int)(blockIdx.x & 7) * per + (int)(blockIdx.x >> 3);
    if (tile >= tiles || (int)(blockIdx.x >> 3) >= per) return;
    const int m0 = tile % tiles_m * kRowsA, n0 = tile / tiles_m * kRowsW;

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
    auto request = [&](int slice) __attribute__((always_inline)) {
        const int buf = slice % kStages * kBuf;
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

    const int wm = (wave & 1) * 32 * TM, wn = (wave >> 1) * 32 * TN, h = lane >> 5, r32 = lane & 31;
    const uint8_t* frag_a = lds + (wm + r32) * kSlice;
    const uint8_t* frag_w = lds + (kRowsA + wn + r32) * kSlice;
    const int swz = (r32 >> 1) & 7;  // (the 32-row blocks start at multiples of 16 rows: the same for all of them)

#pragma unroll
    for (int s = 0; s < kStages - 1; s++)
        if (s < slices) request(s);
    for (int s = 0; s < slices; s++) {
        // requests complete in order: all but the newest slice's have landed
        if (s + 1 < slices) asm volatile("s_waitcnt vmcnt(%0)" ::"n"(kReq * (kStages - 2)) : "memory");
        else asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");
        if (s + kStages - 1 < slices) request(s + kStages - 1);
        const int buf = s % kStages * kBuf;
#pragma unroll
        for (int step = 0; step < 4; step++) {
            const int off = buf + (((2 * step + h) ^ swz) * 16);
            u32x4 fa[TM], fw[TN];
#pragma unroll
            for (int j = 0; j < TM; j++) fa[j] = *reinterpret_cast<const u32x4*>(frag_a + off + j * 32 * kSlice);
#pragma unroll
            for (int i = 0; i < TN; i++) fw[i] = *reinterpret_cast<const u32x4*>(frag_w + off + i * 32 * kSlice);
#pragma unroll
            for (int i = 0; i < TN; i++)
#pragma unroll
                for (int j = 0; j < TM; j++) acc[i][j] = mma<T>(fw[i], fa[j], acc[i][j]);
        }
    }

    // The tile goes through LDS (register x of lane 32 h + n: output row 8 (x / 4) + 4 h + x % 4 of its block, token n), so
    // that the epilogue is one short loop in which a thread has four consecutive outputs of one token and the threads
    // of a wavefront store whole rows of the tile.
    constexpr int kPitch = kRowsW + 4;
    float* tile_c = reinterpret_cast<float*>(lds);
    asm volatile("s_barrier" ::: "memory");  // (every fragment has been read: the products above waited for them)
#pragma unroll
    for (int i = 0; i < TN; i++)
#pragma unroll
        for (int j = 0; j < TM; j++)
#pragma unroll
            for (int g = 0; g < 4; g++)
                *reinterpret_cast<float4*>(tile_c + (wm + 32 * j + r32) * kPitch + wn + 32 * i + 8 * g + 4 * h) =
                    make_float4(acc[i][j][4 * g], acc[i][j][4 * g + 1], acc[i][j][4 * g + 2], acc[i][j][4 * g + 3]);
    __syncthreads();
    constexpr int kQuads = kRowsW / 4;
    const int q4 = 4 * (tid % kQuads), row = n0 + q4;  // (this thread's four rows are the same in every turn)
    if (row >= rows) return;
    int si = -1;
    for (int q = 0; q < out.nseg; q++)
        if (row >= out.seg[q].row0) si = q;
    const skn_dense_seg sg = out.seg[si < 0 ? 0 : si];
    const int left = out.nseg ? sg.row0 + sg.rows - row : out.resid_rows - row;  // rows of the segment from here on
    if (left <= 0 || (out.nseg && si < 0)) return;
    const float4 b = bias ? *reinterpret_cast<const float4*>(bias + row) : make_float4(0.f, 0.f, 0.f, 0.f);
    for (int t = tid / kQuads; t < kRowsA && m0 + t < m; t += 256 / kQuads) {
        const float4 c = *reinterpret_cast<const float4*>(tile_c + t * kPitch + q4);
        float v[4] = {c.x + b.x, c.y + b.y, c.z + b.z, c.w + b.w};
        if (out.nseg == 0) {
            float* p = out.resid + (int64_t)(m0 + t) * out.ldr + row;
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
        const int64_t at = (int64_t)(m0 + t) * sg.ldo + (row - sg.row0);
        if (left >= 4 && sg.out_type == SKN_TYPE_F32) {
            *reinterpret_cast<float4*>((float*)sg.out + at) = make_float4(v[0], v[1], v[2], v[3]);
        } else if (left >= 4) {
            *reinterpret_cast<uint2*>((uint16_t*)sg.out + at) = make_uint2(skn_bf16_bits(v[0]) | ((uint32_t)skn_bf16_bits(v[1]) << 16),
                                                                            skn_bf16_bits(v[2]) | ((uint32_t)skn_bf16_bits(v[3]) << 16));
        } else {
            for (int e = 0; e < left; e++) {
                const float f = e == 0 ? v[0] : e == 1 ? v[1] : v[2];
                if (sg.out_type == SKN_TYPE_F32) ((float*)sg.out)[at + e] = f;
                else ((uint16_t*)sg.out)[at + e] = skn_bf16_bits(f);
            }
        }
    }
}

template <typename T, int TM, int TN>
int launch_gemm(skn_ctx* ctx, const skn_dense_mat& w, const void* a, int lda, int m, const skn_dense_out& out) {
    const int tm = (m + 64 * TM - 1) / (64 * TM), tn = (w.rows + 64 * TN - 1) / (64 * TN), tiles = tm * tn;
    skn_launch(ctx, dense_gemm_kernel<T, TM, TN>, dim3((unsigned)((tiles + 7) / 8 * 8)), dim3(256), (size_t)gemm_lds_bytes<TM, TN>(),
               (const uint8_t*)a, (int64_t)lda * (int64_t)sizeof(T), m, (const uint8_t*)w.w, (int64_t)w.k_pad * (int64_t)sizeof(T), w.rows,
               (int)(w.k_pad * sizeof(T) / kSlice), tm, tiles, w.bias, out);
    SKN_LAUNCH_CHECK(ctx);
    return SKN_OK;
}

template <typename T>
int pick_gemm(skn_ctx* ctx, const skn_dense_mat& w, const void* a, int lda, int m, const skn_dense_out& out) {
    auto tiles = [&](int tm, int tn) { return ((m + 64 * tm - 1) / (64 * tm)) * ((w.rows + 64 * tn - 1) / (64 * tn)); };
    // the largest tile that still gives every compute unit one (three quarters of them: larger tiles move less per product)
    const int enough = ctx->compute_units * 3 / 4;
    if (ctx->opt_dense_tile == 3 || (ctx->opt_dense_tile == 0 && tiles(2, 2) >= enough)) return launch_gemm<T, 2, 2>(ctx, w, a, lda, m, out);
    if (ctx->opt_dense_tile == 2 || (ctx->opt_dense_tile == 0 && tiles(2, 1) >= enough)) return launch_gemm<T, 2, 1>(ctx, w, a, lda, m, out);
    return launch_gemm<T, 1, 1>(ctx, w, a, lda, m, out);
}

template <typename T, int TM, int TN>
int allow_lds(skn_ctx* ctx) {
    SKN_HIP(ctx, hipFuncSetAttribute((const void*)dense_gemm_kernel<T, TM, TN>, hipFuncAttributeMaxDynamicSharedMemorySize, gemm_lds_bytes<TM, TN>()));
    return SKN_OK;
}

int dense_gemm_init(skn_ctx* ctx) {
    SKN_TRY((allow_lds<uint16_t, 2, 2>(ctx)));
    SKN_TRY((allow_lds<uint16_t, 2, 1>(ctx)));
    SKN_TRY((allow_lds<uint16_t, 1, 1>(ctx)));
    SKN_TRY((allow_lds<float, 2, 2>(ctx)));
    SKN_TRY((allow_lds<float, 2, 1>(ctx)));
    SKN_TRY((allow_lds<float, 1, 1>(ctx)));
    return SKN_OK;
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
    SKN_REQUIRE(ctx, out.nseg > 0 || (out.ldr % 4 == 0 && out.resid_rows <= w.rows && ((uintptr_t)out.resid & 15) == 0), SKN_ERR_ARG,
                "dense GEMM: bad residual rows");
    if (w.type == SKN_TYPE_BF16) return pick_gemm<uint16_t>(ctx, w, a, lda, m, out);
    if (w.type == SKN_TYPE_F32) return pick_gemm<float>(ctx, w, a, lda, m, out);
    return skn_fail(ctx, SKN_ERR_TYPE, "dense GEMM: weights of type %d (BF16 or F32)", w.type);
}
