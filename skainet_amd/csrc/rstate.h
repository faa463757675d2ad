// Recurrent state of the linear-attention layers: per sequence and head a matrix [key channel][value channel] in fp32,
// created, zeroed and freed beside the KV cache and carried from token to token.
#pragma once
#include "common.h"

struct skn_rstate {
    int n_seq = 0, heads = 0, dim = 0, dim_pad = 0;
    // element (key channel i, value channel c) of head h at ((seq * heads + h) * dim + c) * dim_pad + i: the key channels
    // of a value channel are contiguous (dim_pad = 32, 64, 128 or 256, zeros from dim on), because value channels are
    // independent of each other and a group of lanes takes one at a time
    float* s = nullptr;
    float* seq_state(int seq) const { return s + (size_t)seq * heads * dim * dim_pad; }
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
