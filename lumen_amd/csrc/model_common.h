// What the models share: turning parameters into device layouts, reading a safetensors file into a model, the turn
// loop over a model's step function, and recording a step as a graph.
#pragma once
#include <functional>
#include <string>
#include <vector>

#include "internal.h"

void f32_to_bf16_host(const float *src, uint16_t *dst, size_t n);
void bf16_to_f32_host(const uint16_t *src, float *dst, size_t n);

// Copies the tensors of a safetensors file that a model names into it, element counts checked (loader.cpp).
int load_safetensors_into(const char *path, const std::vector<std::string> &names, const std::vector<std::vector<int64_t>> &shapes,
                          const std::function<int(const char *, const void *, int, const int64_t *, int)> &set_param,
                          int *n_loaded_out, int *n_missing_out);

// A model as the turn loop sees it (sampler.cpp).  max_len: tokens a sequence may hold.
struct TurnModel {
    int vocab = 0, max_len = 0;
    std::function<int(const int32_t *ids, int n, float *logits_last)> forward;
    std::function<int(int *)> len;
};
int generate_turn(const TurnModel &m, const int32_t *new_tokens, int n_new, const int32_t *history, int n_history,
                  const lumen_sampling *sp, const int32_t *stop_ids, int n_stop, int32_t *out_ids, int out_cap, int *n_out);

// Records what `enqueue` launches on the stream and instantiates it; the stream is synchronised first.
template <typename F>
int record_graph(hipStream_t s, F enqueue, hipGraph_t *graph_out, hipGraphExec_t *exec_out) {
    HIP_TRY(hipStreamSynchronize(s));
    HIP_TRY(hipStreamBeginCapture(s, hipStreamCaptureModeThreadLocal));
    const int rc = enqueue();
    hipGraph_t g = nullptr;
    const hipError_t e = hipStreamEndCapture(s, &g);
    if (rc != LUMEN_OK) {
        if (g) hipGraphDestroy(g);
        return rc;
    }
    if (e != hipSuccess) LUMEN_FAIL(LUMEN_ERR_HIP, "hipStreamEndCapture failed: %s", hipGetErrorString(e));
    const hipError_t ei = hipGraphInstantiate(exec_out, g, nullptr, nullptr, 0);
    if (ei != hipSuccess) {
        hipGraphDestroy(g);
        *exec_out = nullptr;
        LUMEN_FAIL(LUMEN_ERR_HIP, "hipGraphInstantiate failed: %s", hipGetErrorString(ei));
    }
    *graph_out = g;
    return LUMEN_OK;
}
