// Shared by the token-by-token and the chunked form of the linear recurrences
// (linear_scan.hip, chunk_scan.hip): arguments, decays, step sizes.
#pragma once
#include "recurrent.h"

enum ScanMode { kFixed = 0, kStep = 1, kChannel = 2 };

struct ScanArgs {
  float* out;    // [T, H * dv]
  float* state;  // [slots, H, dv, dk]
  const void *q, *k, *v;
  int64_t qs, ks, vs;  // row strides (elements)
  float q_scale, k_scale;
  int qk_rep;          // heads that share a q / k head
  const float* decay;  // kFixed: [H]
  const void* g;       // kStep: step logits [T, H]; kChannel: decay logits [T, H * dk]
  int64_t gs;
  const float* g_bias;  // [H] / [H * dk] or null
  const float* rate;    // kStep: [H]
  const float* skip;    // [H] or null
  float inv_tau;        // kChannel
  const int64_t* pos;
  const int* seq_rows;  // null: row i is sequence i
  const int* slots;
  int n_slots, T, H, dk, dv;
  int min_rows, max_rows;  // sequences with fewer / more rows in the step are another launch's
};

__device__ __forceinline__ float softplusf_(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }

// sigmoid(z)^(1 / tau) = exp(-softplus(-z) / tau).  Only the exponent's absolute error matters, so the
// plain log of 1 + e serves (its error is below 1e-7 where log1p would return e itself).
__device__ __forceinline__ float channel_decay(float z, float inv_tau) {
  const float sp = fmaxf(-z, 0.f) + __logf(1.f + __expf(-fabsf(z)));
  return __expf(-sp * inv_tau);
}

// step size of one (row, head)
template <typename T> __device__ __forceinline__ float step_size(const ScanArgs& g, int64_t row, int h) {
  return softplusf_(ldf<T>((const T*)g.g, row * g.gs + h) + (g.g_bias ? g.g_bias[h] : 0.f));
}

// a sequence with at least this many rows in the step goes through the chunked kernels
constexpr int kChunkMinRows = 8;

bool chunk_scan_ok(int mode, const ScanArgs& g);
void launch_chunk_scan(int mode, const ScanArgs& g, int n_seq, hipStream_t st);
