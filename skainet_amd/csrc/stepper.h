// The decode loop shared by the decoders: the device scalars of a step, the greedy choice of the next token and the
// captured HIP graph that is replayed per token.
//
// A decode step reads every scalar that changes from step to step (token id, position, context length, step index)
// from device memory, so that one captured graph of the step's kernel launches serves every token.  The graph holds
// kernels only (no memset / memcpy nodes).
#pragma once
#include "common.h"

#include <functional>

struct skn_stepper {
    int32_t* state = nullptr;       // [0] token, [1] position, [2] context length, [3] step index
    int32_t* tokens_out = nullptr;  // device array of produced tokens
    int cap = 0;                    // tokens the array holds
    hipGraph_t graph = nullptr;
    hipGraphExec_t graph_exec = nullptr;
    int graph_key = 0;          // the shape the step was captured for (the caller's: its attention split count)
    int graph_generation = -1;  // ctx->opt_generation at capture: every option a step reads, and the stream
};

int skn_stepper_create(skn_ctx* ctx, skn_stepper* s, int cap);
void skn_stepper_free(skn_stepper* s);
void skn_stepper_drop_graph(skn_stepper* s);
// state = {token, pos, pos + 1, 0}
int skn_stepper_set(skn_ctx* ctx, skn_stepper* s, int token, int pos);
// argmax of the logits (first maximum): advance = 1 makes it the next step's token and counts the step, 0 only leaves
// it in tokens_out[0]
int skn_stepper_pick(skn_ctx* ctx, skn_stepper* s, const float* logits, int vocab, int advance);
// Feeds first_token at position pos, then the step's own choice, n_steps times; `step` enqueues one step's launches
// (ending in skn_stepper_pick with advance).  Waits for the tokens.
int skn_stepper_run(skn_ctx* ctx, skn_stepper* s, int first_token, int pos, int n_steps, int key, const std::function<int()>& step,
                    int32_t* tokens_out_host);
