// Dense (bf16 or fp32) weight products with epilogues: the batched GEMM on the matrix cores and the batch-1 matvec.
//
// A dense matrix is several projections of one input stacked along the output axis: [rows, k_pad] row-major, every
// projection starting at a multiple of 32 rows and every row padded with zeros to k_pad, a multiple of 64 elements
// (padding rows are zeros).  What happens to the rows of a projection -- bias, activation, where they go -- is a segment.
#pragma once
#include "common.h"

constexpr int kDenseRowPad = 32, kDenseColPad = 64;
static inline int skn_pad_rows(int n) { return (n + kDenseRowPad - 1) / kDenseRowPad * kDenseRowPad; }
static inline int skn_pad_cols(int k) { return (k + kDenseColPad - 1) / kDenseColPad * kDenseColPad; }

struct skn_dense_mat {
    const void* w = nullptr;
    int type = SKN_TYPE_BF16;     // SKN_TYPE_BF16 or SKN_TYPE_F32
    int rows = 0;                 // stacked rows, a multiple of 32
    int k_pad = 0;                // a multiple of 64
    const float* bias = nullptr;  // [rows] or null
};

// what a segment does to z = W x (+ bias)
enum {
    SKN_OP_NONE = 0,
    SKN_OP_SIGMOID = 1,
    SKN_OP_TANH = 2,
    SKN_OP_DECAY = 3,  // exp(-exp(-1/2) sigmoid(z)): a decay factor between exp(-exp(-1/2)) = 0.545 and 1
    SKN_OP_XIELU = 4,  // p0 z^2 + z / 2 for z > 0, p1 (exp(z) - 1 - z) + z / 2 otherwise
    SKN_OP_GELU = 5,   // z / 2 (1 + tanh(sqrt(2 / pi) (z + 0.044715 z^3)))
};

struct skn_dense_seg {
    int row0, rows;      // stacked rows [row0, row0 + rows)
    int op;
    float p0, p1;
    void* out;           // [m][ldo], row r of the segment at column r
    int ldo;             // a multiple of 4 when m > 1
    int out_type;        // SKN_TYPE_F32, SKN_TYPE_BF16 or (GEMM) SKN_TYPE_F16
};

constexpr int kDenseMaxSegs = 8;
struct skn_dense_out {
    int nseg = 0;
    skn_dense_seg seg[kDenseMaxSegs];
    // residual form (nseg = 0): resid[m][ldr] += mult * (W x + bias) for the first resid_rows rows
    float* resid = nullptr;
    int ldr = 0, resid_rows = 0;
    float mult = 1.f;
    // matvec only: rows of segment cache_seg also go to the key rows of a shared key/value cache, at the position that
    // *pos_dev names (see kv.h)
    int cache_seg = -1;
    void* k_pool = nullptr;
    int elem_type = SKN_TYPE_F16, kv_heads = 0, dim = 0, dim_pad = 0, page_tokens = 0;
    const int32_t* page_table = nullptr;
    const int32_t* pos_dev = nullptr;
    // rows of segment mul_seg are multiplied, after their operation, by a part of their token's row of a table (of
    // mul_type, F32 or BF16): table[tokens[t] * mul_ld + mul_col + row]
    int mul_seg = -1;
    const void* mul_table = nullptr;
    int mul_type = SKN_TYPE_BF16, mul_ld = 0, mul_col = 0;
    const int32_t* mul_tokens = nullptr;
};

// C[m, rows] from A [m][lda] of the matrix's type (lda elements, a multiple of 64, zeros from k to k_pad).
int skn_dense_gemm(skn_ctx* ctx, const skn_dense_mat& w, const void* a, int lda, int m, const skn_dense_out& out);

// The input of a matvec, staged once per workgroup.
enum { SKN_XSRC_PLAIN = 0, SKN_XSRC_GROUP_NORM = 1, SKN_XSRC_MERGE = 2, SKN_XSRC_ADD_NORM = 3 };
struct skn_matvec_src {
    int mode = SKN_XSRC_PLAIN;
    const float* x0 = nullptr;      // columns [0, k0); 16-byte aligned
    int k0 = 0;
    const float* x1 = nullptr;      // columns [off1, off1 + k1), optional
    int off1 = 0, k1 = 0;
    // SKN_XSRC_GROUP_NORM: x0 is divided, in `groups` equal parts, by each part's root mean square, then times norm_w
    const float* norm_w = nullptr;
    int groups = 1;
    float eps = 0.f;
    // SKN_XSRC_ADD_NORM: x = x0 + add / (root mean square of add) * add_w first, then the norm of x in one part.  Every workgroup
    // computes it for itself; x_out, another buffer than x0, receives x
    const float* add = nullptr;
    const float* add_w = nullptr;
    float* x_out = nullptr;
    // SKN_XSRC_MERGE: columns [0, k0) are the heads of a split attention, merged here: x0[split][head][dim_pad]
    // unnormalised outputs, ml[split][head] (maximum in units of log2 e, sum)
    const float* ml = nullptr;
    int splits = 1, heads = 0, dim = 0, dim_pad = 0;
    int sink = 0;                 // 1: one more score, 0, without a value
    const float* gate = nullptr;  // [k0] factors of the merged columns, optional
};
int skn_dense_matvec(skn_ctx* ctx, const skn_dense_mat& w, const skn_matvec_src& src, const skn_dense_out& out);

// ---- row-wise kernels around them (csrc/dense_rows.hip) ----
// y[r] = grouped RMS norm of x[rows ? rows[r] : r]; y of y_type (F32 / BF16), columns width .. ldy zeroed
int skn_group_norm_rows(skn_ctx* ctx, const float* x, int ldx, const int32_t* row_index, const float* w, int n_rows, int width,
                        int groups, float eps, void* y, int ldy, int y_type);
// x[r] += y[r] / rms(y[r]) * y_w; then, with a norm w, h[r] = x[r] / rms(x[r]) * w in h_type (columns width .. ldh zeroed)
int skn_add_norm_rows(skn_ctx* ctx, float* x, int ldx, const float* y, int ldy, const float* y_w, const float* w, int n_rows, int width, float eps,
                      void* h, int ldh, int h_type);
// y[r] = bf16 of x[r], ld columns
int skn_bf16_rows(skn_ctx* ctx, const float* x, int ld, int n_rows, void* y);
// x[r] = scale * table[tokens[r]], with inv_freq (10000^(-2i/width) in double) plus the sinusoid of position pos0_dev[0] + r
int skn_embed_rows(skn_ctx* ctx, const void* table, int table_type, int ld_table, const int32_t* tokens, const int32_t* pos0_dev,
                   const double* inv_freq, float scale, int n_rows, int width, float* x, int ldx);

#ifdef __HIPCC__
__device__ __forceinline__ float skn_sigmoid(float z) { return __builtin_amdgcn_rcpf(1.0f + __expf(-z)); }

// exp(z) - 1 - z for z <= 0: its series near zero, where the difference would cancel (seven terms: 1e-8 at -0.35)
__device__ __forceinline__ float skn_exp_minus_1_minus(float z) {
    const float near0 = 0.5f * z * z *
                        fmaf(z * (1.f / 3), fmaf(z * (1.f / 4), fmaf(z * (1.f / 5), fmaf(z * (1.f / 6), fmaf(z, 1.f / 7, 1.f), 1.f), 1.f), 1.f), 1.f);
    return z > -0.35f ? near0 : __expf(z) - 1.0f - z;
}

__device__ __forceinline__ float skn_xielu_at(float z, float p0, float p1) {
    return fmaf(z > 0.f ? p0 * z : p1, z > 0.f ? z : skn_exp_minus_1_minus(z), 0.5f * z);
}

__device__ __forceinline__ float skn_dense_op(int op, float z, float p0, float p1) {
    switch (op) {
        case SKN_OP_SIGMOID: return skn_sigmoid(z);
        case SKN_OP_TANH: return fmaf(-2.0f, __builtin_amdgcn_rcpf(1.0f + __expf(2.0f * z)), 1.0f);
        case SKN_OP_DECAY: return __expf(-0.60653065971263342f * skn_sigmoid(z));
        case SKN_OP_XIELU: return skn_xielu_at(z, p0, p1);
        case SKN_OP_GELU: return z * skn_sigmoid(z * fmaf(0.0713548162726f, z * z, 1.5957691216057308f));  // 2 sqrt(2 / pi) (1, 0.044715)
        default: return z;
    }
}

// an element of a bf16 or fp32 table
__device__ __forceinline__ float skn_table_at(const void* table, int type, int64_t i) {
    return type == SKN_TYPE_F32 ? ((const float*)table)[i] : __uint_as_float((uint32_t)((const uint16_t*)table)[i] << 16);
}

__device__ __forceinline__ uint16_t skn_bf16_bits(float f) {
    const uint32_t u = __float_as_uint(f);
    if ((u & 0x7FFFFFFFu) > 0x7F800000u) return (uint16_t)((u >> 16) | 0x40u);  // NaN stays NaN
    return (uint16_t)((u + 0x7FFFu + ((u >> 16) & 1u)) >> 16);
}
#endif
