// What the kernels of linear attention share: the forms, the arguments of a call, and the functions of one number that more
// than one of them computes (so that all get the same bits).
#pragma once

#include "common.h"

enum { LA_CONSTANT = 0, LA_FORGET = 1, LA_CHANNEL = 2, LA_MEMORY = 3 };

// The arguments of one call; the same fields in the same order in kernels/ops.py.
struct LaArgs {
  const float* proj;
  int ld, q_off, k_off, v_off;
  const float* decay;              // LA_CONSTANT [H]
  const float *forget_bias, *forget_low;  // LA_FORGET [H * dk]
  int low_off, rank;               // LA_CHANNEL: the low-rank sums' first column and number
  const float *low_up, *low_bias;  // [rank][H * dk], [H * dk]
  float tau;
  int i_off, f_off;                // LA_MEMORY: first columns of the gates' sums
  const float *i_bias, *f_bias;    // [H]
  float cap, q_scale;
  float* state;
  size_t state_stride;
  const int *q_start, *slots, *positions;
  float* rec;    // working memory of steps with longer portions: tk_linear_attention_work_words 32-bit words a token
  float* o;      // [tokens][H][o_head]
  float* floor;  // LA_MEMORY [tokens][H]
  int o_head;
  int n_tokens, n_requests, H, dk, dv, longest;
  // LA_CHANNEL and LA_MEMORY in chunks (n_chunks > 0): every chunk's request and first row, in the requests' order, and every
  // request's first chunk, [n_chunks], [n_chunks], [n_requests + 1]
  const int *chunk_req, *chunk_row0, *first_chunk;
  int n_chunks;
};

__device__ __forceinline__ float la_silu(float x) { return x / (1.0f + expf(-x)); }
__device__ __forceinline__ float la_sigmoid(float x) { return 1.0f / (1.0f + expf(-x)); }
// the forget gate, written out in one multiply-add so that every kernel that computes it gets the same bits
__device__ __forceinline__ float la_forget(float x, float bias, float lo) { return fmaf(1.0f - lo, la_sigmoid(x + bias), lo); }
__device__ __forceinline__ float la_log_sigmoid(float x) { return fminf(x, 0.f) - log1pf(expf(-fabsf(x))); }
__device__ __forceinline__ float la_channel_decay(float z, float tau) { return expf(la_log_sigmoid(z) / tau); }
__device__ __forceinline__ float la_soft_cap(float x, float cap) { return cap * tanhf(x / cap); }

// columns of a head's state: the values', and the keys' sum in the last form
template <int MODE>
__host__ __device__ __forceinline__ int la_columns(int dv) { return MODE == LA_MEMORY ? dv + 1 : dv; }
// where the running maximum after position p of head h is kept
__device__ __forceinline__ size_t la_max_at(const LaArgs& a, int p, int h) {
  return (size_t)a.H * (a.dv + 1) * a.dk + (size_t)(p & 1) * a.H + h;
}

// The gates of LA_MEMORY (linear_attention.hip): gates[t][h] = (decay of the state, or its logarithm; factor on what is written).
void la_launch_gates(const LaArgs& a, float2* gates, int log_decay, hipStream_t stream);
// The chunked form (linear_attention_chunks.hip): whether it takes these sizes, and the call itself.
bool la_chunks_take(int mode, int dk, int longest);
int la_run_chunks(int mode, const LaArgs& a, hipStream_t stream);
