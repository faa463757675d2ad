// The decode loop of csrc/stepper.h.
#include "stepper.h"

namespace {

// state = {token, position, context length, step}
__global__ void set_state_kernel(int32_t* state, int token, int pos) {
    if (threadIdx.x == 0) {
        state[0] = token;
        state[1] = pos;
        state[2] = pos + 1;
        state[3] = 0;
    }
}

// single workgroup: argmax of the logits (first maximum) becomes the next token; the step's scalars advance
__global__ __launch_bounds__(1024) void finish_step_kernel(const float* __restrict__ x, int n, int32_t* state,
                                                           int32_t* __restrict__ tokens_out, int advance) {
    __shared__ float bv[16];
    __shared__ int bi[16];
    float best = -INFINITY;
    int besti = 0x7FFFFFFF;
    auto take = [&](float v, int i) {
        if (v > best || (v == best && i < besti)) {
            best = v;
            besti = i;
        }
    };
    // eight float4 per thread and round, all loaded before the first compare
    const int n4 = n >> 2;
    for (int base = 0; base < n4; base += 8 * 1024) {
        float4 v[8];
#pragma unroll
        for (int j = 0; j < 8; j++) v[j] = reinterpret_cast<const float4*>(x)[min(base + j * 1024 + (int)threadIdx.x, n4 - 1)];
#pragma unroll
        for (int j = 0; j < 8; j++) {
            const int i4 = base + j * 1024 + (int)threadIdx.x;
            if (i4 < n4) {
                take(v[j].x, 4 * i4);
                take(v[j].y, 4 * i4 + 1);
                take(v[j].z, 4 * i4 + 2);
                take(v[j].w, 4 * i4 + 3);
            }
        }
    }
    for (int i = 4 * n4 + threadIdx.x; i < n; i += 1024) take(x[i], i);
    for (int off = 32; off >= 1; off >>= 1) {
        const float ov = __shfl_xor(best, off, 64);
        const int oi = __shfl_xor(besti, off, 64);
        if (ov > best || (ov == best && oi < besti)) {
            best = ov;
            besti = oi;
        }
    }
    if ((threadIdx.x & 63) == 0) {
        bv[threadIdx.x >> 6] = best;
        bi[threadIdx.x >> 6] = besti;
    }
    __syncthreads();
    if (threadIdx.x == 0) {
        for (int w = 1; w < 16; w++)
            if (bv[w] > best || (bv[w] == best && bi[w] < besti)) {
                best = bv[w];
                besti = bi[w];
            }
        const int tok = besti == 0x7FFFFFFF ? 0 : besti;
        if (advance) {
            tokens_out[state[3]] = tok;
            state[0] = tok;
            state[1] += 1;
            state[2] += 1;
            state[3] += 1;
        } else {
            tokens_out[0] = tok;
        }
    }
}

}  // namespace

int skn_stepper_create(skn_ctx* ctx, skn_stepper* s, int cap) {
    s->cap = cap;
    hipError_t e = hipMalloc((void**)&s->state, 4 * sizeof(int32_t));
    if (e == hipSuccess) e = hipMalloc((void**)&s->tokens_out, (size_t)(cap < 4 ? 4 : cap) * sizeof(int32_t));
    if (e != hipSuccess) {
        (void)hipGetLastError();
        return skn_fail(ctx, SKN_ERR_OOM, "decode loop: state of %d tokens: %s", cap, hipGetErrorString(e));
    }
    return SKN_OK;
}

void skn_stepper_drop_graph(skn_stepper* s) {
    if (s->graph_exec) (void)hipGraphExecDestroy(s->graph_exec);
    if (s->graph) (void)hipGraphDestroy(s->graph);
    s->graph_exec = nullptr;
    s->graph = nullptr;
    s->graph_key = 0;
    s->graph_generation = -1;
}

void skn_stepper_free(skn_stepper* s) {
    skn_stepper_drop_graph(s);
    if (s->state) (void)hipFree(s->state);
    if (s->tokens_out) (void)hipFree(s->tokens_out);
    s->state = s->tokens_out = nullptr;
}

int skn_stepper_set(skn_ctx* ctx, skn_stepper* s, int token, int pos) {
    skn_launch(ctx, set_state_kernel, dim3(1), dim3(64), 0, s->state, token, pos);
    SKN_LAUNCH_CHECK(ctx);
    return SKN_OK;
}

int skn_stepper_pick(skn_ctx* ctx, skn_stepper* s, const float* logits, int vocab, int advance) {
    skn_launch(ctx, finish_step_kernel, dim3(1), dim3(1024), 0, logits, vocab, s->state, s->tokens_out, advance);
    SKN_LAUNCH_CHECK(ctx);
    return SKN_OK;
}

int skn_stepper_run(skn_ctx* ctx, skn_stepper* s, int first_token, int pos, int n_steps, int key, const std::function<int()>& step,
                    int32_t* tokens_out_host) {
    SKN_TRY(skn_stepper_set(ctx, s, first_token, pos));
    if (ctx->opt_llama_graph == 0) {
        for (int i = 0; i < n_steps; i++) SKN_TRY(step());
    } else {
        // a captured step has the kernel set of the options (and the stream) it was captured with baked in
        if (s->graph_exec && (s->graph_key != key || s->graph_generation != ctx->opt_generation)) skn_stepper_drop_graph(s);
        if (!s->graph_exec) {
            SKN_HIP(ctx, hipStreamSynchronize(ctx->stream));
            SKN_HIP(ctx, hipStreamBeginCapture(ctx->stream, hipStreamCaptureModeThreadLocal));
            int rc = step();
            hipGraph_t g = nullptr;
            hipError_t e = hipStreamEndCapture(ctx->stream, &g);
            if (rc != SKN_OK) {
                if (g) (void)hipGraphDestroy(g);
                return rc;
            }
            if (e != hipSuccess) return skn_fail(ctx, SKN_ERR_HIP, "stream capture failed: %s", hipGetErrorString(e));
            s->graph = g;
            SKN_HIP(ctx, hipGraphInstantiate(&s->graph_exec, s->graph, nullptr, nullptr, 0));
            s->graph_key = key;
            s->graph_generation = ctx->opt_generation;
            ctx->stat_captures++;
        }
        for (int i = 0; i < n_steps; i++) SKN_HIP(ctx, hipGraphLaunch(s->graph_exec, ctx->stream));
    }
    SKN_HIP(ctx, hipMemcpyAsync(tokens_out_host, s->tokens_out, (size_t)n_steps * sizeof(int32_t), hipMemcpyDeviceToHost, ctx->stream));
    SKN_HIP(ctx, hipStreamSynchronize(ctx->stream));
    return SKN_OK;
}
