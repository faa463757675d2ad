// Paged KV cache object shared by the cache kernels, decode attention and the decoder.
#pragma once
#include "common.h"

// what the pools hold
enum {
    SKN_KV_PLAIN = 0,   // fp16 keys and values
    SKN_KV_SHARED = 1,  // rows that are key and value (skn_kv_create_shared)
    SKN_KV_RANGED = 2,  // keys and values of their own sizes (skn_kv_create_ranged)
    SKN_KV_LATENT = 3,  // a latent and a rotated key part per token (skn_kv_create_latent)
};

struct skn_kv {
    int kind = SKN_KV_PLAIN;
    int n_seq = 0, n_head = 0, head_dim = 0, page_tokens = 0, max_tokens = 0;
    int pages_per_seq = 0, n_pages = 0;
    // page p, head h, slot s, element e lives at ((p * n_head + h) * page_tokens + s) * head_dim + e:
    // one head's tokens of a page are contiguous, so attention streams page_tokens * head_dim * 2 bytes runs.
    uint16_t* k_pool = nullptr;
    uint16_t* v_pool = nullptr;
    // A shared cache (skn_kv_create_shared) holds one row per token and head, the projected key before its norm: it is the
    // value as it stands, and times the token's key_scale (the norm's reciprocal root mean square, over all heads) the key.
    // Its rows are fp16 or fp32 (elem_type), dim elements and zeros up to head_dim = 64, 128 or 256; v_pool is null.
    // A ranged cache holds keys of dim and values of vdim elements, both in rows of head_dim = 64, 128 or 256.
    // A latent cache holds one row per token: vdim elements of the latent, then the rotated key part, dim elements in all and
    // zeros up to head_dim = 128 x 1, 2, 3, 5 or 8; v_pool is null.
    int elem_type = SKN_TYPE_F16, dim = 0, vdim = 0;
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

// ---- attention over a range of the cache (csrc/attention_ranged.hip; parameters: skn_ranged_attn of the header) ----
// The keys that position i sees: all before it, a window, or its chunk.
struct skn_range {
    int kind = SKN_MASK_CAUSAL, size = 0;
#ifdef __HIPCC__
    __host__ __device__
#endif
    int first(int i) const { return kind == SKN_MASK_WINDOW ? (i + 1 > size ? i + 1 - size : 0) : kind == SKN_MASK_CHUNK ? i - i % size : 0; }
};
// the longest range that a position below max_ctx sees
int skn_range_longest(const skn_range& r, int max_ctx);
// Rows of a prompt, as skn_shared_prep_rows / skn_shared_attn_rows: q, k, v [n][ld*] projected with bias; gate [n][ldg] factors of
// the output, optional.
int skn_ranged_prep_rows(skn_ctx* ctx, skn_kv* kv, int seq, const skn_ranged_attn& p, const float* q, int ldq, const float* k, int ldk, const float* v,
                         int ldv, int n, int pos0, float* q_prep);
int skn_ranged_attn_rows(skn_ctx* ctx, skn_kv* kv, int seq, const skn_ranged_attn& p, const float* q_prep, int n, int pos0, const float* gate, int ldg,
                         void* out, int ldo, int out_type);
// One token from its projections, its norms, rotation and cache rows included.  n_splits > 1: unmerged partials without sink and gate.
int skn_ranged_attn_step(skn_ctx* ctx, skn_kv* kv, int seq, const skn_ranged_attn& p, const float* q, const float* k, const float* v, const float* gate,
                         const int32_t* state_dev, int n_splits, float* opart, float* ml, float* out);
int skn_ranged_splits(skn_ctx* ctx, int n_head, int streams, const skn_range& r, int max_ctx);

// ---- attention over latents (csrc/attention_latent.hip; parameters: skn_latent_attn of the header) ----
// Scratch of a prompt's expanded keys and values, grown on demand and owned by the caller.
struct skn_latent_ws {
    void* mem = nullptr;
    size_t bytes = 0;
};
// n rows at pos0 .. of sequence seq: q [n][ldq], d [n][ldd] (latent and rotated part, before norm and rotation; null: the rows
// are in the cache already), out [n][ldo].
int skn_latent_rows(skn_ctx* ctx, skn_kv* kv, int seq, const skn_latent_attn& p, const float* q, int ldq, const float* d, int ldd, int n, int pos0,
                    float* q_prep, float* lat, skn_latent_ws* ws, void* out, int ldo, int out_type);
// floats per row that skn_latent_rows needs in q_prep and in lat
size_t skn_latent_prep_floats(const skn_kv* kv, const skn_latent_attn& p);
size_t skn_latent_lat_floats(const skn_kv* kv, const skn_latent_attn& p);
// One token.  q_prep, opart (16 splits) as many floats as skn_latent_prep_floats says, ml 32 per head.
int skn_latent_step(skn_ctx* ctx, skn_kv* kv, int seq, const skn_latent_attn& p, const float* q, const float* d, const int32_t* state_dev, int n_splits,
                    float* q_prep, float* opart, float* ml, float* out);
int skn_latent_splits(skn_ctx* ctx, const skn_kv* kv, const skn_latent_attn& p, int max_ctx);
// the matrix-core forms for prompts (csrc/attention_prefill.hip): fp16
struct skn_prefill_ranged {
    skn_range range;
    float scale = 0.f, softcap = 0.f;
    int sink = 0, vdim = 0;
    const float* gate = nullptr;
    int ldg = 0;
    void* out = nullptr;
    int ldo = 0, out_type = SKN_TYPE_F32;
};
bool skn_ranged_prefill_fits(const skn_kv* kv);
int skn_ranged_prefill_launch(skn_ctx* ctx, skn_kv* kv, int seq, const float* q_prep, int n_queries, int pos0, int n_head, const skn_prefill_ranged& p);
// padded key width for heads of dim + rot_dim and vdim elements, 0: no such form
int skn_latent_prefill_width(int dim, int rot_dim, int vdim);
// k [tokens][ldk] (dim per head), rot [tokens][rot_dim] and v [tokens][ldv], fp16, of the tokens from token0 (a multiple of 32) on
int skn_latent_prefill_launch(skn_ctx* ctx, const uint16_t* k, int ldk, const uint16_t* rot, const uint16_t* v, int ldv, int dim, int rot_dim, int token0,
                              const float* q_prep, int n_queries, int pos0, int n_head, const skn_prefill_ranged& p);
