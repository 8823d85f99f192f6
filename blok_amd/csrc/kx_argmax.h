// kx_argmax.h -- greedy sampling: lowest-index argmax of rows of logits (kx_argmax.hip).
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>

constexpr int KX_ARGMAX_PARTS = 64;  // workgroups per row, and partials per row in the scratch
#define KX_ARGMAX_SCRATCH_FLOATS(tokens) ((size_t)(tokens) * 2 * KX_ARGMAX_PARTS)
// scratch: KX_ARGMAX_SCRATCH_FLOATS(tokens) floats
int kx_argmax_launch(const float *logits, int tokens, int n, int stride, uint32_t *out, float *scratch, hipStream_t st);
