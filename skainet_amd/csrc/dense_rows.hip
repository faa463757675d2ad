// Row-wise kernels around the dense products: RMS norm in groups, the sum of a normed row with the norm that follows, and the
// embedding, scaled or with sinusoidal positions.
#include "dense.h"

namespace {

constexpr int kMaxGroups = 1024;

// one workgroup per row; LDS: the row, then one factor per group
__global__ __launch_bounds__(256) void group_norm_kernel(const float* __restrict__ x, int ldx, const int32_t* __restrict__ row_index,
                                                         const float* __restrict__ w, int width, int groups, float eps, void* __restrict__ y, int ldy,
                                                         int y_type) {
    extern __shared__ float lds[];
    __shared__ float part[4];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, gs = width / groups;
    const float* xr = x + (int64_t)(row_index ? row_index[blockIdx.x] : (int)blockIdx.x) * ldx;
    float* factor = lds + width;
    float ss = 0.f;
    for (int i = tid; i < width; i += 256) {
        const float v = xr[i];
        lds[i] = v;
        ss = fmaf(v, v, ss);
    }
    if (groups == 1) {  // the whole workgroup sums
        ss = wave_sum(ss);
        if (lane == 0) part[wave] = ss;
        __syncthreads();
        if (tid == 0) factor[0] = 1.0f / sqrtf(((part[0] + part[1]) + (part[2] + part[3])) / (float)gs + eps);
    } else {
        __syncthreads();
        for (int g = wave; g < groups; g += 4) {
            float s = 0.f;
            for (int i = lane; i < gs; i += 64) s = fmaf(lds[g * gs + i], lds[g * gs + i], s);
            s = wave_sum(s);
            if (lane == 0) factor[g] = 1.0f / sqrtf(s / (float)gs + eps);
        }
    }
    __syncthreads();
    const float inv_gs = 1.0f / (float)gs;
    for (int i = tid; i < ldy; i += 256) {
        float v = 0.f;
        if (i < width) v = lds[i] * factor[(int)(((float)i + 0.5f) * inv_gs)] * w[i];
        if (y_type == SKN_TYPE_F32) ((float*)y)[(int64_t)blockIdx.x * ldy + i] = v;
        else ((uint16_t*)y)[(int64_t)blockIdx.x * ldy + i] = skn_bf16_bits(v);
    }
}

// The angle is formed and reduced modulo 2 pi in double (as the rotary embedding's is).
__global__ __launch_bounds__(256) void embed_kernel(const void* __restrict__ table, int table_type, int ld_table,
                                                    const int32_t* __restrict__ tokens, const int32_t* __restrict__ pos0_dev,
                                                    const double* __restrict__ inv_freq, float scale, int width, float* __restrict__ x, int ldx) {
    const int row = blockIdx.x, pos = pos0_dev[0] + row;
    const int64_t at = (int64_t)tokens[row] * ld_table;
    for (int i = blockIdx.y * 256 + threadIdx.x; 2 * i < width; i += gridDim.y * 256) {
        float sn = 0.f, cs = 0.f;
        if (inv_freq) skn_rope_sincos_freq(pos, inv_freq[i], &sn, &cs);
#pragma unroll
        for (int e = 0; e < 2; e++) {
            const int col = 2 * i + e;
            if (col >= width) continue;
            x[(int64_t)row * ldx + col] = fmaf(scale, skn_table_at(table, table_type, at + col), e ? cs : sn);
        }
    }
}

// one workgroup per row; LDS: the row
__global__ __launch_bounds__(256) void add_norm_kernel(float* __restrict__ x, int ldx, const float* __restrict__ y, int ldy, const float* __restrict__ y_w,
                                                       const float* __restrict__ w, int width, float eps, void* __restrict__ h, int ldh, int h_type) {
    extern __shared__ float lds[];
    __shared__ float part[8];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    float* xr = x + (int64_t)blockIdx.x * ldx;
    const float* yr = y + (int64_t)blockIdx.x * ldy;
    auto inv_rms = [&](float ss, float* red) {
        ss = wave_sum(ss);
        if (lane == 0) red[wave] = ss;
        __syncthreads();
        return 1.0f / sqrtf(((red[0] + red[1]) + (red[2] + red[3])) / (float)width + eps);
    };
    float ss = 0.f;
    for (int i = tid; i < width; i += 256) {
        const float v = yr[i];
        lds[i] = v;
        ss = fmaf(v, v, ss);
    }
    const float ry = inv_rms(ss, part);
    ss = 0.f;
    for (int i = tid; i < width; i += 256) {  // (a thread's own elements throughout)
        const float v = xr[i] + lds[i] * ry * y_w[i];
        xr[i] = v;
        lds[i] = v;
        ss = fmaf(v, v, ss);
    }
    if (!w) return;
    const float rx = inv_rms(ss, part + 4);
    for (int i = tid; i < ldh; i += 256) {
        const float v = i < width ? lds[i] * rx * w[i] : 0.f;
        if (h_type == SKN_TYPE_F32) ((float*)h)[(int64_t)blockIdx.x * ldh + i] = v;
        else ((uint16_t*)h)[(int64_t)blockIdx.x * ldh + i] = skn_bf16_bits(v);
    }
}

__global__ __launch_bounds__(256) void bf16_rows_kernel(const float4* __restrict__ x, int64_t n, uint2* __restrict__ y) {
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= n) return;
    const float4 v = x[i];
    y[i] = make_uint2(skn_bf16_bits(v.x) | ((uint32_t)skn_bf16_bits(v.y) << 16), skn_bf16_bits(v.z) | ((uint32_t)skn_bf16_bits(v.w) << 16));
}

__global__ void xielu_kernel(const float* __restrict__ z, int64_t n, float p0, float p1, float* __restrict__ out) {
    const int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
    if (i < n) out[i] = skn_xielu_at(z[i], p0, p1);
}

__global__ void gelu_kernel(const float* __restrict__ z, int64_t n, float* __restrict__ out) {
    const int64_t i = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
    if (i < n) out[i] = skn_dense_op(SKN_OP_GELU, z[i], 0.f, 0.f);
}

}  // namespace

int skn_group_norm_rows(skn_ctx* ctx, const float* x, int ldx, const int32_t* row_index, const float* w, int n_rows, int width, int groups, float eps,
                        void* y, int ldy, int y_type) {
    SKN_REQUIRE(ctx, groups > 0 && groups <= kMaxGroups && width % groups == 0, SKN_ERR_SHAPE,
                "norm: %d columns in %d groups (equal groups, at most %d)", width, groups, kMaxGroups);
    const size_t lds = (size_t)(width + groups) * sizeof(float);
    SKN_REQUIRE(ctx, lds <= 64000, SKN_ERR_SHAPE, "norm: rows of %d columns (at most %d)", width, 64000 / 4 - groups);
    skn_launch(ctx, group_norm_kernel, dim3(n_rows), dim3(256), lds, x, ldx, row_index, w, width, groups, eps, y, ldy, y_type);
    SKN_LAUNCH_CHECK(ctx);
    return SKN_OK;
}

int skn_add_norm_rows(skn_ctx* ctx, float* x, int ldx, const float* y, int ldy, const float* y_w, const float* w, int n_rows, int width, float eps,
                      void* h, int ldh, int h_type) {
    SKN_REQUIRE(ctx, width > 0 && width <= 16000, SKN_ERR_SHAPE, "norm: rows of %d columns (at most 16000)", width);
    skn_launch(ctx, add_norm_kernel, dim3(n_rows), dim3(256), (size_t)width * sizeof(float), x, ldx, y, ldy, y_w, w, width, eps, h, ldh, h_type);
    SKN_LAUNCH_CHECK(ctx);
    return SKN_OK;
}

int skn_bf16_rows(skn_ctx* ctx, const float* x, int ld, int n_rows, void* y) {
    SKN_REQUIRE(ctx, ld % 4 == 0, SKN_ERR_SHAPE, "bf16 rows: pitch %d is no multiple of 4", ld);
    const int64_t quads = (int64_t)n_rows * ld / 4;
    skn_launch(ctx, bf16_rows_kernel, dim3((unsigned)((quads + 255) / 256)), dim3(256), 0, (const float4*)x, quads, (uint2*)y);
    SKN_LAUNCH_CHECK(ctx);
    return SKN_OK;
}

int skn_embed_rows(skn_ctx* ctx, const void* table, int table_type, int ld_table, const int32_t* tokens, const int32_t* pos0_dev,
                   const double* inv_freq, float scale, int n_rows, int width, float* x, int ldx) {
    // (a single row: its columns over several workgroups)
    const int split = n_rows == 1 ? (width + 511) / 512 : 1;
    skn_launch(ctx, embed_kernel, dim3(n_rows, split), dim3(256), 0, table, table_type, ld_table, tokens, pos0_dev, inv_freq, scale, width, x, ldx);
    SKN_LAUNCH_CHECK(ctx);
    return SKN_OK;
}

extern "C" {

int skn_rmsnorm_grouped(skn_ctx* ctx, const float* x_dev, const float* w_dev, int rows, int n, int groups, float eps, float* y_dev) {
    SKN_REQUIRE(nullptr, ctx != nullptr, SKN_ERR_ARG, "skn_rmsnorm_grouped: ctx is null");
    SKN_REQUIRE(ctx, rows >= 0 && n > 0, SKN_ERR_ARG, "skn_rmsnorm_grouped: bad shape");
    if (rows == 0) return SKN_OK;
    SKN_REQUIRE(ctx, x_dev && w_dev && y_dev, SKN_ERR_ARG, "skn_rmsnorm_grouped: null pointer");
    return skn_group_norm_rows(ctx, x_dev, n, nullptr, w_dev, rows, n, groups, eps, y_dev, n, SKN_TYPE_F32);
}

int skn_xielu(skn_ctx* ctx, const float* z_dev, int64_t n, float pos, float neg, float* out_dev) {
    SKN_REQUIRE(nullptr, ctx != nullptr, SKN_ERR_ARG, "skn_xielu: ctx is null");
    SKN_REQUIRE(ctx, n >= 0, SKN_ERR_ARG, "skn_xielu: negative size");
    if (n == 0) return SKN_OK;
    SKN_REQUIRE(ctx, z_dev && out_dev, SKN_ERR_ARG, "skn_xielu: null pointer");
    skn_launch(ctx, xielu_kernel, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, z_dev, n, pos, neg, out_dev);
    SKN_LAUNCH_CHECK(ctx);
    return SKN_OK;
}

int skn_gelu(skn_ctx* ctx, const float* z_dev, int64_t n, float* out_dev) {
    SKN_REQUIRE(nullptr, ctx != nullptr, SKN_ERR_ARG, "skn_gelu: ctx is null");
    SKN_REQUIRE(ctx, n >= 0, SKN_ERR_ARG, "skn_gelu: negative size");
    if (n == 0) return SKN_OK;
    SKN_REQUIRE(ctx, z_dev && out_dev, SKN_ERR_ARG, "skn_gelu: null pointer");
    skn_launch(ctx, gelu_kernel, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, z_dev, n, out_dev);
    SKN_LAUNCH_CHECK(ctx);
    return SKN_OK;
}

}  // extern "C"
