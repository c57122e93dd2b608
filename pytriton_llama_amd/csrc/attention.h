// What the attention kernels share beside their tables: which keys a query sees, and what is done
// to a row's result.
//
// A query at position p sees the keys at positions j <= p for which
//   window > 0   p - j < window (its own key and the window - 1 before it), or j < keep_first
//   chunk > 0    j / chunk == p / chunk (chunks of so many positions, counted from position 0)
//   neither      all of them
// (window and chunk exclude each other; keep_first goes with a window).
//
// sink (or null): one float a query head; the softmax denominator of that head holds exp(sink) once
// more, a term without key and value that is not scaled. gate (or null): one float a row and query
// head (row * gate_stride + head); the head's result is multiplied by sigmoid(gate).
//
// softcap > 0: a scaled score s becomes softcap * tanh(s / softcap) before the mask and the softmax.
#pragma once
#include "common.h"
#include <math.h>

struct AttnExtras {
  int window, keep_first, chunk;
  const float* sink;
  const float* gate;
  long gate_stride;
  float softcap;
};

// The first key that a query at position pos sees (of the window, for a window that keeps the
// sequence's first keys as well).
__device__ __forceinline__ int first_seen(const AttnExtras& ex, int pos) {
  if (ex.window > 0) return max(0, pos - ex.window + 1);
  if (ex.chunk > 0) return max(0, pos) / ex.chunk * ex.chunk;
  return 0;
}

__device__ __forceinline__ float head_gate(const AttnExtras& ex, int row, int head) {
  return ex.gate ? 1.0f / (1.0f + expf(-ex.gate[(size_t)row * ex.gate_stride + head])) : 1.0f;
}

__device__ __forceinline__ float cap_score(const AttnExtras& ex, float s) {
  return ex.softcap > 0.f ? ex.softcap * tanhf(s / ex.softcap) : s;
}

// tanh from the hardware's exp2 and reciprocal: 1 - 2 / (1 + e^(2x)), with x2 = 2 x log2 e. Absolute
// error of a few 1e-7 (the result feeds the exponent of a softmax); saturates to -1 and 1.
__device__ __forceinline__ float tanh_exp2(float x2) {
  return fmaf(-2.0f, __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(x2)), 1.0f);
}

static inline bool extras_ok(const AttnExtras& ex) {
  return ex.softcap >= 0.f && !(ex.chunk > 0 && (ex.window > 0 || ex.keep_first > 0));
}
