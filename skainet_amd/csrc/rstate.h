// Recurrent state of the linear-attention layers: per sequence and head a matrix [key channel][value channel] in fp32,
// created, zeroed and freed beside the KV cache and carried from token to token.
#pragma once
#include "common.h"

struct skn_rstate {
    int n_seq = 0, heads = 0, dim = 0, vdim = 0, dim_pad = 0;
    // element (key channel i < dim, value channel c < vdim) of head h at ((seq * heads + h) * vdim + c) * dim_pad + i: the key channels
    // of a value channel are contiguous (dim_pad = 32, 64, 128 or 256, zeros from dim on), because value channels are
    // independent of each other and a group of lanes takes one at a time
    float* s = nullptr;
    float* seq_state(int seq) const { return s + (size_t)seq * heads * vdim * dim_pad; }
    // States with convolutions (skn_rstate_create_conv) also hold the inputs of the last `taps` tokens, a ring by position: channel
    // c of position p at (seq * taps + p % taps) * channels + c; channels are q, k [kv_heads * dim] and v [heads * vdim].
    int kv_heads = 0, taps = 0, channels = 0;
    float* conv = nullptr;
    std::vector<int> pos;  // host: tokens absorbed per sequence (skn_gated_delta; a decoder brings its own positions)
    float* seq_conv(int seq) const { return conv + (size_t)seq * taps * channels; }
};

// ---- generalized delta rule (csrc/delta.hip) ----
//   S_t = diag(w_t) S_{t-1} - (a_t u_t) (u_t^T S_{t-1}) + k_t v_t^T,   o_t = S_t^T r_t,   u = k / sqrt(sum k^2 + 1e-6)
// Rows of a prompt: r, k, v, w, a fp32 [n][ld], heads x dim columns; pack: skn_delta_pack_floats(n) floats of scratch.
// o [n][heads * dim].
size_t skn_delta_pack_floats(const skn_rstate* st, int n);
int skn_delta_rows(skn_ctx* ctx, skn_rstate* st, int seq, const float* r, const float* k, const float* v, const float* w, const float* a, int ld, int n,
                   float* pack, float* o);
// y[n][ldy] (F32 or BF16) = o / rms over each head * norm * g   (g [n][ldg])
int skn_delta_gate_rows(skn_ctx* ctx, const float* o, const float* g, int ldg, const float* norm, int n, int heads, int dim, float eps, void* y, int ldy,
                        int y_type);
// One token, everything after its projections: the decay from its low-rank input t [rank] (w2 [heads * dim][rank_pad] of
// w2_type, b2 [heads * dim]), the state's step, norm and gate.  r, k, v, a, g [heads * dim]; y [heads * dim].
struct skn_delta_step {
    const float *r, *k, *v, *a, *g, *t;
    const void* w2;
    int w2_type, rank, rank_pad;
    const float* b2;
    const float* norm;
    float eps;
    float* y;
};
int skn_delta_step_launch(skn_ctx* ctx, skn_rstate* st, int seq, const skn_delta_step& p);

// ---- gated delta rule with a decay per key channel (csrc/gated_delta.hip; equations: skn_channel_delta of the header) ----
// Rows of a prompt at positions pos0 ..: q, k, v before their convolutions, beta and z, all [n][ld]; cq, ck, cv [n][ld] scratch for
// what the convolutions leave; pack: skn_gated_delta_pack_floats(n) floats of scratch.  o [n][heads * vdim].
size_t skn_gated_delta_pack_floats(const skn_rstate* st, int n);
int skn_gated_delta_rows(skn_ctx* ctx, skn_rstate* st, int seq, const skn_channel_delta& p, const float* q, const float* k, const float* v, const float* beta,
                         const float* z, int ld, int n, int pos0, float* cq, float* ck, float* cv, float* pack, float* o);
// One token, everything after its projections: convolutions, z and the output's gate from their low-rank inputs, the state's step,
// norm and gate.  beta: after its sigmoid.
struct skn_gated_step {
    const float *q, *k, *v, *beta;
    const float *a_low, *g_low;  // [rank_a_pad], [rank_g_pad]: finite beyond the ranks
    const void *w_a, *w_g;       // [heads * dim][rank_a_pad], [heads * vdim][rank_g_pad] of w_type
    int w_type, rank_a_pad, rank_g_pad;
    const float* bias_a;  // [heads * dim]
    const float* norm;    // [heads * vdim]
    float eps;
    const int32_t* state;  // the step's position at [1]
    float* y;              // [heads * vdim]
};
int skn_gated_step_launch(skn_ctx* ctx, skn_rstate* st, int seq, const skn_channel_delta& c, const skn_gated_step& p);
