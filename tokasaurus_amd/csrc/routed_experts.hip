// A feed-forward made of many small gated experts of which a token uses a few, and the
// per-head products of a mixer whose heads share a latent.  T is the storage type of weights
// and activations; sums are 32-bit, and the router is 32-bit arithmetic throughout.
//
//   tk_expert_route      per token: logits over all experts, their softmax or sigmoids, choice by score
//                        (+ correction) inside the best groups of neighbouring experts, the chosen
//                        experts' scores as weights; optionally the sigmoid gate of a shared expert
//   tk_expert_lookup     the chosen experts from tables by token id, for all layers of a step at once
//   tk_expert_gate_up    per (token, chosen expert): act(W_gate h) * (W_up h), of h or of weight * h, or the form with clamps
//   tk_expert_combine    per token: sum of weight * W_down(...) over its experts, weight * h for an
//                        identity expert, plus gate * (a shared expert's output)
//   tk_head_linear       y[t, h, :] = W[h] x[t, h, :]: one matrix a head; optionally the leading part of a
//                        head turned instead of multiplied, or the result times a sigmoid gate per element
//   tk_squared_relu      x <- max(x, 0)^2, in place
//
// These kernels compute a row (a token, a pair) independently of every other row, with sums
// in an order that the sizes alone fix: a token's result does not depend on its batch.
#include <math.h>

#include "common.h"

// Sum over i < n of w[i] * x[i], the lanes of a wavefront taking pieces of 16 bytes in turn when
// both rows allow, single elements otherwise; every lane returns the sum.
template <typename T>
__device__ __forceinline__ float wave_dot(const T* __restrict__ w, const T* __restrict__ x, int n) {
  constexpr int V = 16 / sizeof(T);
  const int lane = threadIdx.x & (TK_WAVE - 1);
  float acc = 0.f;
  if (n % V == 0 && (((uintptr_t)w | (uintptr_t)x) & 15) == 0) {
    for (int i = lane * V; i < n; i += TK_WAVE * V) {
      const uint4 wa = *(const uint4*)(w + i), xa = *(const uint4*)(x + i);
      const T* wp = (const T*)&wa;
      const T* xp = (const T*)&xa;
#pragma unroll
      for (int e = 0; e < V; ++e) acc = fmaf(to_f32<T>(wp[e]), to_f32<T>(xp[e]), acc);
    }
  } else {
    for (int i = lane; i < n; i += TK_WAVE) acc = fmaf(to_f32<T>(w[i]), to_f32<T>(x[i]), acc);
  }
  return wave_sum(acc);
}

// The same for two rows of weights against one x, in one pass (each sum in the order wave_dot has).
template <typename T>
__device__ __forceinline__ void wave_dot2(const T* __restrict__ w0, const T* __restrict__ w1, const T* __restrict__ x, int n,
                                          float& d0, float& d1) {
  constexpr int V = 16 / sizeof(T);
  const int lane = threadIdx.x & (TK_WAVE - 1);
  float a0 = 0.f, a1 = 0.f;
  if (n % V == 0 && (((uintptr_t)w0 | (uintptr_t)w1 | (uintptr_t)x) & 15) == 0) {
    for (int i = lane * V; i < n; i += TK_WAVE * V) {
      const uint4 wa = *(const uint4*)(w0 + i), wb = *(const uint4*)(w1 + i), xa = *(const uint4*)(x + i);
      const T* wp = (const T*)&wa;
      const T* wq = (const T*)&wb;
      const T* xp = (const T*)&xa;
#pragma unroll
      for (int e = 0; e < V; ++e) {
        a0 = fmaf(to_f32<T>(wp[e]), to_f32<T>(xp[e]), a0);
        a1 = fmaf(to_f32<T>(wq[e]), to_f32<T>(xp[e]), a1);
      }
    }
  } else {
    for (int i = lane; i < n; i += TK_WAVE) {
      a0 = fmaf(to_f32<T>(w0[i]), to_f32<T>(x[i]), a0);
      a1 = fmaf(to_f32<T>(w1[i]), to_f32<T>(x[i]), a1);
    }
  }
  d0 = wave_sum(a0);
  d1 = wave_sum(a1);
}

// --------------------------------------------------------------------------
// The router.  One workgroup a token.  n_all = routed + identity experts.  ids [tokens, top] names
// the chosen experts in the order of their choice scores, weights [tokens, top] their scores: softmax, or
// SIGMOID, each the sigmoid of its own logit (the correction, where there is one, moves the choice, not the weight;
// without one sigmoid scores are ranked by their logits, which order them without saturating); with `norm_scale` != 0 the chosen scores divided by
// their sum (+ 1e-20) and multiplied by norm_scale.  Without `w_gate` a given `shared_gate` is filled with ones.
// --------------------------------------------------------------------------
template <typename T, bool SIGMOID>
__global__ __launch_bounds__(1024) void expert_route_kernel(
    const T* __restrict__ h, int h_stride, const T* __restrict__ w_router, const float* __restrict__ correction,
    const T* __restrict__ w_gate, int width, int n_all, int groups, int keep, int top, int* __restrict__ ids,
    float* __restrict__ weights, float* __restrict__ shared_gate, float norm_scale) {
  extern __shared__ float sm[];
  float* score = sm;                 // [n_all] logits, then softmax scores
  float* choice = sm + n_all;        // [n_all] score + correction, -inf outside the kept groups and once taken
  float* mark = sm + 2 * n_all;      // [groups]
  const int t = blockIdx.x;
  const int lane = threadIdx.x & (TK_WAVE - 1), wave = threadIdx.x / TK_WAVE, nwaves = blockDim.x / TK_WAVE;
  const T* row = h + (size_t)t * h_stride;
  if (!w_gate && shared_gate && threadIdx.x == 0) shared_gate[t] = 1.f;
  for (int e = wave; e < n_all + (w_gate ? 1 : 0); e += nwaves) {
    const float d = wave_dot<T>(e < n_all ? w_router + (size_t)e * width : w_gate, row, width);
    if (lane == 0) {
      if (e < n_all) score[e] = d;
      else shared_gate[t] = 1.0f / (1.0f + expf(-d));
    }
  }
  __syncthreads();
  if (wave != 0) return;  // the rest is the work of one wavefront, whose lanes hand over through LDS in its own order
  if (SIGMOID) {
    for (int e = lane; e < n_all; e += TK_WAVE) {
      const float z = score[e], s = 1.0f / (1.0f + expf(-z));
      score[e] = s;
      choice[e] = correction ? s + correction[e] : z;
    }
  } else {
    float m = -INFINITY;
    for (int e = lane; e < n_all; e += TK_WAVE) m = fmaxf(m, score[e]);
    m = wave_max(m);
    float sum = 0.f;
    for (int e = lane; e < n_all; e += TK_WAVE) {
      const float x = expf(score[e] - m);
      score[e] = x;
      sum += x;
    }
    sum = wave_sum(sum);
    for (int e = lane; e < n_all; e += TK_WAVE) {
      const float s = score[e] / sum;
      score[e] = s;
      choice[e] = correction ? s + correction[e] : s;
    }
  }
  wave_sync();
  if (keep < groups) {
    const int per = n_all / groups;
    for (int g = lane; g < groups; g += TK_WAVE) {
      float best = -INFINITY;
      for (int e = g * per; e < (g + 1) * per; ++e) best = fmaxf(best, choice[e]);
      mark[g] = best;
    }
    wave_sync();
    for (int g = lane; g < groups; g += TK_WAVE) {
      int ahead = 0;  // groups that come before this one: a larger mark, or an equal one further left
      const float mine = mark[g];
      for (int o = 0; o < groups; ++o) ahead += (mark[o] > mine || (mark[o] == mine && o < g)) ? 1 : 0;
      if (ahead >= keep)
        for (int e = g * per; e < (g + 1) * per; ++e) choice[e] = -INFINITY;
    }
    wave_sync();
  }
  // the `top` largest choices, ties to the left; with up to 64 experts a lane's choice stays in a register
  const bool few = n_all <= TK_WAVE;
  float mine = few && lane < n_all ? choice[lane] : -INFINITY;
  float sum = 0.f;
  for (int r = 0; r < top; ++r) {
    float best = -INFINITY;
    int at = 0x7fffffff;
    if (few) {
      best = mine;
      at = mine > -INFINITY ? lane : 0x7fffffff;
    } else {
      for (int e = lane; e < n_all; e += TK_WAVE) {
        const float c = choice[e];
        if (c > best) { best = c; at = e; }
      }
    }
#pragma unroll
    for (int o = TK_WAVE / 2; o > 0; o >>= 1) {
      const float ob = __shfl_xor(best, o, TK_WAVE);
      const int oa = __shfl_xor(at, o, TK_WAVE);
      if (ob > best || (ob == best && oa < at)) { best = ob; at = oa; }
    }
    if (at == 0x7fffffff) at = -1;  // fewer open experts than places: the place stays empty
    const float w = at >= 0 ? score[at] : 0.f;
    sum += w;
    if (lane == 0) {
      ids[(size_t)t * top + r] = at;
      weights[(size_t)t * top + r] = w;
      if (at >= 0 && !few) choice[at] = -INFINITY;
    }
    if (few) {
      if (lane == at) mine = -INFINITY;
    } else {
      wave_sync();
    }
  }
  if (norm_scale != 0.f && lane == 0)  // (the lane reads back what it wrote)
    for (int r = 0; r < top; ++r) weights[(size_t)t * top + r] = weights[(size_t)t * top + r] / (sum + 1e-20f) * norm_scale;
}

TK_API int tk_expert_route(int dt, const void* h, int h_stride, const void* w_router, const float* correction,
                           const void* w_gate, int tokens, int width, int n_all, int groups, int keep, int top,
                           int* ids, float* weights, float* shared_gate, float norm_scale, int sigmoid, hipStream_t stream) {
  TK_REQUIRE(tokens >= 0 && width > 0 && n_all > 0 && groups > 0 && n_all % groups == 0 && keep > 0 && keep <= groups &&
                 top > 0 && top <= n_all,
             "expert_route: bad sizes tokens=%d width=%d experts=%d groups=%d keep=%d top=%d", tokens, width, n_all,
             groups, keep, top);
  TK_REQUIRE(h && w_router && ids && weights && (!w_gate || shared_gate) && h_stride >= width,
             "expert_route: a pointer is missing or the row stride is too short");
  const size_t smem = sizeof(float) * (size_t)(2 * n_all + groups);
  TK_REQUIRE(smem <= 48 * 1024, "expert_route: %d experts do not fit the local memory", n_all);
  if (tokens == 0) return 0;
  // a wavefront a logit where the step has few tokens (each dot product is a chain of loads), four wavefronts for many
  const int threads = tokens <= 64 ? 1024 : 256;
#define ER_LAUNCH(T, S)                                                                                                       \
  hipLaunchKernelGGL((expert_route_kernel<T, S>), dim3(tokens), dim3(threads), smem, stream, (const T*)h, h_stride,            \
                     (const T*)w_router, correction, (const T*)w_gate, width, n_all, groups, keep, top, ids, weights, shared_gate, \
                     norm_scale)
  if (dt == TK_F32) {
    if (sigmoid) ER_LAUNCH(float, true); else ER_LAUNCH(float, false);
  } else {
    if (sigmoid) ER_LAUNCH(bf16_t, true); else ER_LAUNCH(bf16_t, false);
  }
#undef ER_LAUNCH
  TK_CHECK_LAUNCH("expert_route");
  return 0;
}

// --------------------------------------------------------------------------
// Experts by token id: for every layer with such a table, table[layer] [vocab][tops[layer]], the row of every token of the
// step, ids[layer] [tokens][tops[layer]] (the layers' parts begin `at[layer]` * tokens numbers apart).  An id below 0 names
// an entry of `last_token`, as in the embedding.  One launch a step for all layers: the choice rests on the ids alone.
// --------------------------------------------------------------------------
struct LookupLayer {
  const int* table;
  int top, at;
};
__global__ __launch_bounds__(256) void expert_lookup_kernel(const int* __restrict__ token_ids, const int* __restrict__ last_token, int vocab,
                                                            const LookupLayer* __restrict__ layers, int* __restrict__ ids, int tokens) {
  const int t = blockIdx.x * blockDim.x + threadIdx.x;
  if (t >= tokens) return;
  const LookupLayer l = layers[blockIdx.y];
  int id = token_ids[t];
  if (id < 0) id = last_token[-id - 1];
  id = min(max(id, 0), vocab - 1);
  for (int k = 0; k < l.top; ++k) ids[(size_t)l.at * tokens + (size_t)t * l.top + k] = l.table[(size_t)id * l.top + k];
}

TK_API int tk_expert_lookup(const int* token_ids, const int* last_token, int vocab, const void* layers, int* ids, int n_layers, int tokens,
                            hipStream_t stream) {
  TK_REQUIRE(token_ids && layers && ids && vocab > 0 && n_layers > 0 && n_layers < 65536 && tokens >= 0, "expert_lookup: bad arguments");
  if (tokens == 0) return 0;
  hipLaunchKernelGGL(expert_lookup_kernel, dim3((tokens + 255) / 256, n_layers), dim3(256), 0, stream, token_ids, last_token, vocab,
                     (const LookupLayer*)layers, ids, tokens);
  TK_CHECK_LAUNCH("expert_lookup");
  return 0;
}

// --------------------------------------------------------------------------
// inter[pair, j] = silu(W_gate[e] h)_j * (W_up[e] h)_j for pair = (token, place), e = ids[pair] a routed
// expert (others are skipped).  w_gate_up: [experts][2 * ff][width], gate rows first.  `in_weights` (null or a number
// a pair): the expert reads in_weights[pair] * h; the products being linear, the factor goes on their 32-bit sums.
// `limit` > 0: the activation with clamps instead (clamped_glu of common.h).
// Workgroup (pair, block of EX_ROWS outputs), a wavefront an output at a time.
// --------------------------------------------------------------------------
#define EX_ROWS 4  // one output a wavefront: a step of few tokens is a chain of loads, so many short workgroups
template <typename T>
__global__ __launch_bounds__(256) void expert_gate_up_kernel(
    const T* __restrict__ h, int h_stride, const T* __restrict__ w_gate_up, const int* __restrict__ ids,
    const float* __restrict__ in_weights, T* __restrict__ inter, int width, int ff, int experts, int top, float limit, float alpha) {
  const int pair = blockIdx.x;
  const int e = ids[pair];
  if (e < 0 || e >= experts) return;
  const int lane = threadIdx.x & (TK_WAVE - 1), wave = threadIdx.x / TK_WAVE, nwaves = blockDim.x / TK_WAVE;
  const T* row = h + (size_t)(pair / top) * h_stride;
  const T* wg = w_gate_up + (size_t)e * 2 * ff * width;
  const T* wu = wg + (size_t)ff * width;
  const int j0 = blockIdx.y * EX_ROWS;
  for (int j = j0 + wave; j < min(j0 + EX_ROWS, ff); j += nwaves) {
    float g, u;
    wave_dot2<T>(wg + (size_t)j * width, wu + (size_t)j * width, row, width, g, u);
    if (lane == 0) {
      if (in_weights) {
        g *= in_weights[pair];
        u *= in_weights[pair];
      }
      if (limit > 0.f) {
        inter[(size_t)pair * ff + j] = from_f32<T>(clamped_glu<T>(g, u, limit, alpha));
        continue;
      }
      // gate, up and the activation as the storage type sees them, as the dense feed-forward's epilogue
      const float gr = round_to<T>(g), ur = round_to<T>(u);
      const float a = round_to<T>(gr / (1.0f + expf(-gr)));
      inter[(size_t)pair * ff + j] = from_f32<T>(a * ur);
    }
  }
}

TK_API int tk_expert_gate_up(int dt, const void* h, int h_stride, const void* w_gate_up, const int* ids, const float* in_weights, void* inter,
                             int tokens, int width, int ff, int experts, int top, float limit, float alpha, hipStream_t stream) {
  TK_REQUIRE(tokens >= 0 && width > 0 && ff > 0 && experts > 0 && top > 0 && h_stride >= width,
             "expert_gate_up: bad sizes tokens=%d width=%d ff=%d experts=%d top=%d", tokens, width, ff, experts, top);
  TK_REQUIRE(h && w_gate_up && ids && inter, "expert_gate_up: a pointer is missing");
  if (tokens == 0) return 0;
  const dim3 grid(tokens * top, (ff + EX_ROWS - 1) / EX_ROWS);
  TK_REQUIRE(grid.y < 65536, "expert_gate_up: an expert of %d rows is too large", ff);
  if (dt == TK_F32)
    hipLaunchKernelGGL(expert_gate_up_kernel<float>, grid, dim3(256), 0, stream, (const float*)h, h_stride,
                       (const float*)w_gate_up, ids, in_weights, (float*)inter, width, ff, experts, top, limit, alpha);
  else
    hipLaunchKernelGGL(expert_gate_up_kernel<bf16_t>, grid, dim3(256), 0, stream, (const bf16_t*)h, h_stride,
                       (const bf16_t*)w_gate_up, ids, in_weights, (bf16_t*)inter, width, ff, experts, top, limit, alpha);
  TK_CHECK_LAUNCH("expert_gate_up");
  return 0;
}

// --------------------------------------------------------------------------
// out[t, c] = sum over the places k of token t, in order, of
//     weights[t, k] * (W_down[e] inter[t, k])_c       e = ids[t, k] a routed expert
//     weights[t, k] * h[t, c]                         e an identity expert (e >= experts)
// plus shared_gate[t] * shared[t, c] when a shared expert's output is given.  out is 32-bit.  `unit` != 0: a routed
// expert's output is added as it is (its weight went on what it read).  weights null: equal parts, 1 / top each.
// w_down: [experts][width][ff].  Workgroup (token, block of EX_ROWS columns).
// --------------------------------------------------------------------------
template <typename T>
__global__ __launch_bounds__(256) void expert_combine_kernel(
    const T* __restrict__ h, int h_stride, const T* __restrict__ inter, const T* __restrict__ w_down,
    const int* __restrict__ ids, const float* __restrict__ weights, const float* __restrict__ shared,
    const float* __restrict__ shared_gate, float* __restrict__ out, int width, int ff, int experts, int top, int unit) {
  const int t = blockIdx.x;
  const int lane = threadIdx.x & (TK_WAVE - 1), wave = threadIdx.x / TK_WAVE, nwaves = blockDim.x / TK_WAVE;
  const int c0 = blockIdx.y * EX_ROWS;
  for (int c = c0 + wave; c < min(c0 + EX_ROWS, width); c += nwaves) {
    float acc = 0.f;
    for (int k = 0; k < top; ++k) {
      const int e = ids[(size_t)t * top + k];
      if (e < 0) continue;
      const float g = unit && e < experts ? 1.f : (weights ? weights[(size_t)t * top + k] : 1.0f / (float)top);
      float y;
      if (e < experts)
        y = round_to<T>(wave_dot<T>(w_down + ((size_t)e * width + c) * ff, inter + ((size_t)t * top + k) * ff, ff));
      else
        y = to_f32<T>(h[(size_t)t * h_stride + c]);
      acc = fmaf(g, y, acc);
    }
    if (shared) acc = fmaf(shared_gate[t], shared[(size_t)t * width + c], acc);
    if (lane == 0) out[(size_t)t * width + c] = acc;
  }
}

TK_API int tk_expert_combine(int dt, const void* h, int h_stride, const void* inter, const void* w_down, const int* ids,
                             const float* weights, const float* shared, const float* shared_gate, float* out, int tokens,
                             int width, int ff, int experts, int top, int unit, hipStream_t stream) {
  TK_REQUIRE(tokens >= 0 && width > 0 && ff > 0 && experts > 0 && top > 0 && h_stride >= width,
             "expert_combine: bad sizes tokens=%d width=%d ff=%d experts=%d top=%d", tokens, width, ff, experts, top);
  TK_REQUIRE(h && inter && w_down && ids && out && (!shared || shared_gate), "expert_combine: a pointer is missing");
  if (tokens == 0) return 0;
  const dim3 grid(tokens, (width + EX_ROWS - 1) / EX_ROWS);
  TK_REQUIRE(grid.y < 65536, "expert_combine: a width of %d is too large", width);
  if (dt == TK_F32)
    hipLaunchKernelGGL(expert_combine_kernel<float>, grid, dim3(256), 0, stream, (const float*)h, h_stride,
                       (const float*)inter, (const float*)w_down, ids, weights, shared, shared_gate, out, width, ff,
                       experts, top, unit);
  else
    hipLaunchKernelGGL(expert_combine_kernel<bf16_t>, grid, dim3(256), 0, stream, (const bf16_t*)h, h_stride,
                       (const bf16_t*)inter, (const bf16_t*)w_down, ids, weights, shared, shared_gate, out, width, ff,
                       experts, top, unit);
  TK_CHECK_LAUNCH("expert_combine");
  return 0;
}

// --------------------------------------------------------------------------
// y[t, hd * n_out + o] = sum_i W[hd][o][i] * x[t, hd * n_in + i]: a matrix a head.  y is T or 32-bit.
// Workgroup (token, head, block of HL_ROWS outputs).
// `rot` > 0 (for a matrix whose leading rot x rot block is the identity, with zeros beside and below it): the leading
// rot outputs of a head are its leading inputs turned by position * freq[i], pairs (i, i + rot/2) with `pair_half` and
// (2i, 2i + 1) without, cosine and sine times rot_scale, rounded as the inputs are.
// `gate` (or null): y[t, hd * n_out + o] is multiplied by sigmoid(gate[t, hd * n_out + o]) before its one rounding.
// --------------------------------------------------------------------------
#define HL_ROWS 32
template <typename T>
struct HeadExtra {
  const int* positions;
  const float* freq;
  int rot, pair_half;
  float rot_scale;
  const T* gate;
  int gate_stride;
};
template <typename T, typename O>
__global__ __launch_bounds__(256) void head_linear_kernel(const T* __restrict__ x, int x_stride, const T* __restrict__ w,
                                                          O* __restrict__ y, int y_stride, int n_in, int n_out, HeadExtra<T> ex) {
  const int t = blockIdx.x, hd = blockIdx.y;
  const int lane = threadIdx.x & (TK_WAVE - 1), wave = threadIdx.x / TK_WAVE, nwaves = blockDim.x / TK_WAVE;
  const T* row = x + (size_t)t * x_stride + (size_t)hd * n_in;
  const T* wh = w + (size_t)hd * n_out * n_in;
  O* dst = y + (size_t)t * y_stride + (size_t)hd * n_out;
  const int o0 = blockIdx.z * HL_ROWS;
  if (o0 < ex.rot) {  // this block's turned outputs, a thread a pair that begins here
    const int half = ex.rot / 2;
    for (int i = threadIdx.x; i < half; i += blockDim.x) {
      const int e0 = ex.pair_half ? i : 2 * i, e1 = ex.pair_half ? i + half : 2 * i + 1;
      if (e0 < o0 || e0 >= o0 + HL_ROWS) continue;
      float sn, cs, u = to_f32<T>(row[e0]), v = to_f32<T>(row[e1]);
      sincosf(__fmul_rn((float)ex.positions[t], ex.freq[i]), &sn, &cs);
      rotate_pair(u, v, cs * ex.rot_scale, sn * ex.rot_scale, u, v);
      dst[e0] = from_f32<O>(round_to<T>(u));
      dst[e1] = from_f32<O>(round_to<T>(v));
    }
  }
  for (int o = max(o0, ex.rot) + wave; o < min(o0 + HL_ROWS, n_out); o += nwaves) {
    float d = wave_dot<T>(wh + (size_t)o * n_in, row, n_in);
    if (lane == 0) {
      if (ex.gate) d /= 1.0f + expf(-to_f32<T>(ex.gate[(size_t)t * ex.gate_stride + (size_t)hd * n_out + o]));
      dst[o] = from_f32<O>(d);
    }
  }
}

TK_API int tk_head_linear(int dt, const void* x, int x_stride, const void* w, void* y, int y_stride, int out_f32,
                          int tokens, int heads, int n_in, int n_out, const int* positions, const float* freq, int rot,
                          int pair_half, float rot_scale, const void* gate, int gate_stride, hipStream_t stream) {
  TK_REQUIRE(tokens >= 0 && heads > 0 && n_in > 0 && n_out > 0 && x_stride >= heads * n_in && y_stride >= heads * n_out,
             "head_linear: bad sizes tokens=%d heads=%d in=%d out=%d strides %d %d", tokens, heads, n_in, n_out, x_stride,
             y_stride);
  TK_REQUIRE(x && w && y, "head_linear: a pointer is missing");
  TK_REQUIRE(rot >= 0 && rot % 2 == 0 && rot <= n_in && rot <= n_out && (rot == 0 || (positions && freq)),
             "head_linear: %d turned elements of heads of %d and %d", rot, n_in, n_out);
  TK_REQUIRE(!gate || gate_stride >= heads * n_out, "head_linear: the gate's rows are too short");
  if (tokens == 0) return 0;
  const dim3 grid(tokens, heads, (n_out + HL_ROWS - 1) / HL_ROWS);
  TK_REQUIRE(grid.y < 65536 && grid.z < 65536, "head_linear: too many heads or outputs");
  const HeadExtra<float> ef{positions, freq, rot, pair_half, rot_scale, (const float*)gate, gate_stride};
  const HeadExtra<bf16_t> eb{positions, freq, rot, pair_half, rot_scale, (const bf16_t*)gate, gate_stride};
  if (dt == TK_F32)
    hipLaunchKernelGGL((head_linear_kernel<float, float>), grid, dim3(256), 0, stream, (const float*)x, x_stride,
                       (const float*)w, (float*)y, y_stride, n_in, n_out, ef);
  else if (out_f32)
    hipLaunchKernelGGL((head_linear_kernel<bf16_t, float>), grid, dim3(256), 0, stream, (const bf16_t*)x, x_stride,
                       (const bf16_t*)w, (float*)y, y_stride, n_in, n_out, eb);
  else
    hipLaunchKernelGGL((head_linear_kernel<bf16_t, bf16_t>), grid, dim3(256), 0, stream, (const bf16_t*)x, x_stride,
                       (const bf16_t*)w, (bf16_t*)y, y_stride, n_in, n_out, eb);
  TK_CHECK_LAUNCH("head_linear");
  return 0;
}

// --------------------------------------------------------------------------
// x <- max(x, 0)^2 in place.
// --------------------------------------------------------------------------
template <typename T>
__global__ void squared_relu_kernel(T* __restrict__ x, size_t n) {
  const size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (i < n) {
    const float v = fmaxf(to_f32<T>(x[i]), 0.f);
    x[i] = from_f32<T>(v * v);
  }
}

TK_API int tk_squared_relu(int dt, void* x, size_t n, hipStream_t stream) {
  if (n == 0) return 0;
  const size_t blocks = (n + 255) / 256;
  TK_REQUIRE(x && blocks < (1u << 31), "squared_relu: bad arguments");
  if (dt == TK_F32)
    hipLaunchKernelGGL(squared_relu_kernel<float>, dim3((unsigned)blocks), dim3(256), 0, stream, (float*)x, n);
  else
    hipLaunchKernelGGL(squared_relu_kernel<bf16_t>, dim3((unsigned)blocks), dim3(256), 0, stream, (bf16_t*)x, n);
  TK_CHECK_LAUNCH("squared_relu");
  return 0;
}
