// Paged KV cache object shared by the cache kernels, decode attention and the decoder.
#pragma once
#include "common.h"

struct skn_kv {
    int n_seq = 0, n_head = 0, head_dim = 0, page_tokens = 0, max_tokens = 0;
    int pages_per_seq = 0, n_pages = 0;
    // page p, head h, slot s, element e lives at ((p * n_head + h) * page_tokens + s) * head_dim + e:
    // one head's tokens of a page are contiguous, so attention streams page_tokens * head_dim * 2 bytes runs.
    uint16_t* k_pool = nullptr;
    uint16_t* v_pool = nullptr;
    // A shared cache (skn_kv_create_shared) holds one row per token and head, the projected key before its norm: it is the
    // value as it stands, and times the token's key_scale (the norm's reciprocal root mean square, over all heads) the key.
    // Its rows are fp16 or fp32 (elem_type), dim elements and zeros up to head_dim = 64, 128 or 256; v_pool is null.
    bool shared = false;
    int elem_type = SKN_TYPE_F16, dim = 0;
    float* key_scale = nullptr;  // [page][slot]
    int32_t* page_table_dev = nullptr;  // [n_seq][pages_per_seq], -1 = not mapped
    int32_t* len_dev = nullptr;         // [n_seq] tokens held, the kernels' source of append positions
    int32_t* nctx_dev = nullptr;        // [n_seq] staging for explicit attention lengths
    int* ticket_dev = nullptr;          // workgroups of an append launch count themselves in (zero between launches)
    std::vector<int32_t> page_table;    // host mirror
    std::vector<int32_t> len;           // host mirror
    std::vector<int32_t> free_pages;    // stack of unmapped page ids
    std::vector<int32_t> nctx_host;     // keeps explicit attention lengths alive while their upload is queued
};

// Maps pages so that sequence `seq` can hold `new_len` tokens; uploads new table entries on the stream.
int skn_kv_reserve(skn_ctx* ctx, skn_kv* kv, int seq, int new_len);

// Counts n more tokens into a sequence whose rows were written by a kernel outside the cache code (pages reserved
// by the caller): host mirror and device length.
int skn_kv_advance_len(skn_ctx* ctx, skn_kv* kv, int seq, int n);

// Attention over `kv` with per-sequence lengths taken from a device array; max_ctx bounds them (host knowledge).
int skn_attn_launch(skn_ctx* ctx, skn_kv* kv, const float* q_dev, const int32_t* nctx_dev, int max_ctx, float scale,
                    float* out_dev);
int skn_attn_launch_ex(skn_ctx* ctx, skn_kv* kv, const float* q_dev, const int32_t* nctx_dev, int n_queries,
                       int seq_fixed, int n_splits, float* partial, int* counters, float scale, float* out_dev,
                       int n_q_head = 0);  // query heads (a multiple of the cached heads; 0: as many)
int skn_attn_splits(skn_ctx* ctx, int pairs, int max_ctx);
// Causal attention of n_queries rows of one sequence: row t attends to its first first_ctx + t tokens (head_dim 64 / 128).
int skn_attn_prefill_launch(skn_ctx* ctx, skn_kv* kv, int seq, const float* q_dev, int n_queries, int first_ctx, float scale,
                            float* out_dev, int n_q_head = 0);

// ---- attention over a shared cache (csrc/attention_shared.hip; parameters: skn_shared_attn of the header) ----
// Rows of a prompt: q [n][n_head * dim] (pitch ldq) and k [n][kv heads * dim] (pitch ldk), projected with bias, of tokens at
// positions pos0 .. of sequence seq: normalises them, q with its temperature to q_prep [n][n_head][head_dim], k to the
// cache (pages reserved by the caller; lengths are not advanced).
int skn_shared_prep_rows(skn_ctx* ctx, skn_kv* kv, int seq, const skn_shared_attn& p, const float* q, int ldq, const float* k, int ldk, int n,
                         int pos0, float* q_prep);
// out[n][ldo] (F32 or BF16): causal attention of the prepared rows, row t over the first pos0 + t + 1 tokens
int skn_shared_attn_rows(skn_ctx* ctx, skn_kv* kv, int seq, const skn_shared_attn& p, const float* q_prep, int n, int pos0, void* out, int ldo,
                         int out_type);
// One token: q [n_head * dim] and k [kv heads * dim] projected, the cache row already stored (the matvec's cache segment);
// state_dev: device {token, position, context length, ...}.  n_splits == 1: out [n_head * dim] fp32; otherwise the
// unmerged partials opart[split][head][head_dim] and ml[split][head] (maximum in units of log2 e, sum).
int skn_shared_attn_step(skn_ctx* ctx, skn_kv* kv, int seq, const skn_shared_attn& p, const float* q, const float* k, const int32_t* state_dev,
                         int n_splits, float* opart, float* ml, float* out);
int skn_shared_attn_splits(skn_ctx* ctx, const skn_kv* kv, int n_head, int max_ctx);
// the matrix-core form for prompts (csrc/attention_prefill.hip): fp16 caches, head_dim 64 or 128
int skn_shared_attn_prefill_launch(skn_ctx* ctx, skn_kv* kv, int seq, const float* q_prep, int n_queries, int first_ctx, int n_head, float scale,
                                   void* out, int ldo, int out_type);
