// Linear attention with a decay, as a recurrence over the tokens of each request, and what stands
// around it in the mixers that use it: the short causal convolution that is added to a mixer's input,
// the norm of the recurrence's result (head by head or over all heads) with an optional gate,
// and a sigmoid gate on the rows of another mixer.
//
// Per head, with a matrix S [dk][dv] kept per request in 32-bit:
//     S_t = diag(a_t) S_(t-1) + k_t v_t^T        o_t = S_t^T q_t
// in four forms, all read from the 32-bit sums `proj` of one stacked product:
//   LA_CONSTANT  q = silu(.), k = silu(.), v = silu(.), a_t = decay[head] for every row and token
//   LA_FORGET    q = silu(.), f = low + (1 - low) * sigmoid(. + bias) per head and row of S; a_t = f, k_t = 1 - f; v as it is
//   LA_CHANNEL   q = q_scale * ., k and v as they are; a_t = sigmoid(z)^(1 / tau) per head and row of S, z = up low + bias
//                with `low` some of the sums (a projection of low rank, whose second matrix is applied here)
//   LA_MEMORY    q = q_scale * ., k and v as they are; two numbers a head and token, i = cap tanh((. + i_bias) / cap) and
//                f = log sigmoid(cap tanh((. + f_bias) / cap)); with a running maximum m' = max(f + m, i) from m = 0, kept
//                per head beside S: a_t = exp(f + m - m') and exp(i - m') k_t v_t^T is what is written.  One column more,
//                dv, whose value is always 1, sums the keys (n); its read-out n . q and exp(-m') (`floor`) leave beside o.
// Everything from the sums on (activations, gates, the state, the read-out) is 32-bit arithmetic.
//
// The state row of a slot is [H][columns][dk]: a column's dk numbers lie together; behind them, in the last form, [2][H]
// running maxima: the one after position p lies in row p % 2, so that workgroups that take the same token need no order
// among themselves.  The columns of S
// do not meet: a column is owned by LA_LANES neighbouring lanes that cut dk between them and add up through the
// wavefront's own data paths, always in the same order, so a token's result does not depend on how its request's
// tokens were cut into steps or on what shares the batch (the running maxima of a portion are combined in an order of
// its own: they change a result by rounding only).  Longer portions of the last two forms go in chunks of products on the
// matrix cores instead, with the same 32-bit sums in another order: linear_attention_chunks.hip.
#include "linear_attention.h"

#define LA_LANES 16
#define LA_COLS 4      // columns a wavefront owns
#define LA_WAVES 8     // most wavefronts of a workgroup (they share nothing: a workgroup is only a unit of dispatch)

// A row of `rec`: [q: H x dkp | k or f: H x dkp | (LA_CHANNEL) a: H x dkp | v: H x columns, padded to a multiple of 4],
// dkp = dk rounded up to 64 times the pieces a lane holds, zeros in the padding (a padded row of S meets a zero of q).
template <int MODE>
__host__ __device__ __forceinline__ int la_value_at(int H, int dkp) { return (MODE == LA_CHANNEL ? 3 : 2) * H * dkp; }
template <int MODE>
__host__ __device__ __forceinline__ int la_rec_width(int H, int dkp, int dv) {
  return la_value_at<MODE>(H, dkp) + (H * la_columns<MODE>(dv) + 3) / 4 * 4;
}
// --------------------------------------------------------------------------
// Before the recurrence, once a token: the activations, into rows that the recurrence's lanes read 16 bytes at a time
// (LA_CHANNEL: without the decays).
// --------------------------------------------------------------------------
template <int MODE>
__global__ __launch_bounds__(256) void linear_attention_prepare_kernel(LaArgs a, int dkp) {
  const size_t t = blockIdx.y;
  const int x = blockIdx.x * blockDim.x + threadIdx.x;
  const int ld_rec = la_rec_width<MODE>(a.H, dkp, a.dv), v_at = la_value_at<MODE>(a.H, dkp);
  if (x >= ld_rec) return;
  const float* row = a.proj + t * a.ld;
  float val = 0.f;
  if (x < 2 * a.H * dkp) {
    const int which = x / (a.H * dkp), rem = x % (a.H * dkp), h = rem / dkp, i = rem % dkp;
    if (i < a.dk) {
      const int c = h * a.dk + i;
      if (MODE == LA_CHANNEL || MODE == LA_MEMORY) {
        val = which == 0 ? row[a.q_off + c] * a.q_scale : row[a.k_off + c];
      } else if (which == 0) {
        val = la_silu(row[a.q_off + c]);
      } else if (MODE == LA_CONSTANT) {
        val = la_silu(row[a.k_off + c]);
      } else {
        val = la_forget(row[a.k_off + c], a.forget_bias[c], a.forget_low[c]);
      }
    }
  } else if (x < v_at) {
    return;  // (the decays: the kernel below)
  } else {
    const int c = x - v_at;
    if (MODE == LA_MEMORY) {
      const int h = c / (a.dv + 1), i = c % (a.dv + 1);
      if (h < a.H) val = i < a.dv ? row[a.v_off + h * a.dv + i] : 1.f;
    } else if (c < a.H * a.dv) {
      val = MODE == LA_CONSTANT ? la_silu(row[a.v_off + c]) : row[a.v_off + c];
    }
  }
  a.rec[t * ld_rec + x] = val;
}

// The decays of LA_CHANNEL into `rec`: a thread one channel of LA_TOKENS neighbouring tokens, which share the loads of
// the second matrix.
#define LA_TOKENS 8
__global__ __launch_bounds__(256) void linear_attention_decay_kernel(LaArgs a, int dkp) {
  const int x = blockIdx.x * blockDim.x + threadIdx.x;
  if (x >= a.H * dkp) return;
  const int h = x / dkp, i = x % dkp, t0 = blockIdx.y * LA_TOKENS, n = min(LA_TOKENS, a.n_tokens - t0);
  const int ld_rec = la_rec_width<LA_CHANNEL>(a.H, dkp, a.dv);
  float* dst = a.rec + (size_t)t0 * ld_rec + 2 * a.H * dkp + x;
  if (i >= a.dk) {
    for (int j = 0; j < n; ++j) dst[(size_t)j * ld_rec] = 0.f;
    return;
  }
  const int c = h * a.dk + i, width = a.H * a.dk;
  float z[LA_TOKENS];
#pragma unroll
  for (int j = 0; j < LA_TOKENS; ++j) z[j] = 0.f;
  for (int r = 0; r < a.rank; ++r) {
    const float w = a.low_up[(size_t)r * width + c];
#pragma unroll
    for (int j = 0; j < LA_TOKENS; ++j) z[j] = fmaf(a.proj[(size_t)(t0 + min(j, n - 1)) * a.ld + a.low_off + r], w, z[j]);
  }
#pragma unroll
  for (int j = 0; j < LA_TOKENS; ++j)
    if (j < n) dst[(size_t)j * ld_rec] = la_channel_decay(z[j] + a.low_bias[c], a.tau);
}

// The gates of LA_MEMORY for every token of a (head, request): LA_GATES tokens at a time as a scan.  A token takes the
// maximum from m to max(m + F, M) with F = f and M = i; two tokens one after the other are such a step again, with
// F = F1 + F2 and M = max(M1 + F2, M2).  gates[t][h] = (decay of the state, factor on what is written), floor[t][h] = exp(-m).
// With `log_decay` the decay's logarithm is stored.
#define LA_GATES 512
__global__ __launch_bounds__(LA_GATES) void linear_attention_gates_kernel(LaArgs a, float2* __restrict__ gates, int log_decay) {
  __shared__ float sum_f[LA_GATES / TK_WAVE], top_i[LA_GATES / TK_WAVE], carry;
  const int h = blockIdx.x, r = blockIdx.y;
  const int first = a.q_start[r], last = a.q_start[r + 1];
  if (first >= last) return;
  float* slot = a.state + (size_t)a.slots[r] * a.state_stride;
  const int lane = threadIdx.x & (TK_WAVE - 1), wave = threadIdx.x / TK_WAVE;
  const int p0 = a.positions[first];
  float m_in = p0 > 0 ? slot[la_max_at(a, p0 - 1, h)] : 0.f;
  float raw_i = 0.f, raw_f = 0.f;
  auto ask = [&](int t) {
    if (t < last) {
      raw_i = a.proj[(size_t)t * a.ld + a.i_off + h];
      raw_f = a.proj[(size_t)t * a.ld + a.f_off + h];
    }
  };
  ask(first + threadIdx.x);
  for (int t0 = first; t0 < last; t0 += LA_GATES) {
    const int t = t0 + threadIdx.x;
    const bool in = t < last;
    const float gi = in ? la_soft_cap(raw_i + a.i_bias[h], a.cap) : -INFINITY;
    const float gf = in ? la_log_sigmoid(la_soft_cap(raw_f + a.f_bias[h], a.cap)) : 0.f;
    ask(t + LA_GATES);
    float F = gf, M = gi;
#pragma unroll
    for (int o = 1; o < TK_WAVE; o <<= 1) {
      const float f_up = __shfl_up(F, o, TK_WAVE), m_up = __shfl_up(M, o, TK_WAVE);
      if (lane >= o) {
        M = fmaxf(m_up + F, M);
        F = f_up + F;
      }
    }
    if (lane == TK_WAVE - 1) {
      sum_f[wave] = F;
      top_i[wave] = M;
    }
    __syncthreads();
    float m_wave = m_in;  // the maximum in front of this wavefront's tokens
    for (int w = 0; w < wave; ++w) m_wave = fmaxf(m_wave + sum_f[w], top_i[w]);
    const float m = fmaxf(m_wave + F, M);
    float m_prev = __shfl_up(m, 1, TK_WAVE);
    if (lane == 0) m_prev = m_wave;
    if (in) {
      const float ld = gf + m_prev - m;
      gates[(size_t)t * a.H + h] = make_float2(log_decay ? ld : expf(ld), expf(gi - m));
      a.floor[(size_t)t * a.H + h] = expf(-m);
      if (t == last - 1) slot[la_max_at(a, a.positions[t], h)] = m;
    }
    if (threadIdx.x == LA_GATES - 1) carry = m;
    __syncthreads();
    m_in = carry;
  }
}

// --------------------------------------------------------------------------
// The recurrence.  A wavefront owns LA_COLS columns of one (head, request); the wavefronts of a workgroup take
// neighbouring blocks of columns and share nothing (a step of single tokens is a launch of thousands of short
// wavefronts, which are dispatched faster in workgroups of several).  A column of S is
// owned by LA_LANES neighbouring lanes; lane l holds rows 4 * (l + LA_LANES * n) + e, n < NQ, e < 4, so that it reads
// its pieces of q and of k (or f) as whole 16-byte loads.  Nothing is staged in LDS and there is no barrier: the
// wavefronts of a head read the same rows of `rec` (served by the caches), PF tokens ahead of the arithmetic.
//   LA_CONSTANT  s = a s + k v      LA_FORGET  s = f s + (1 - f) v = v + f (s - v)      LA_CHANNEL  s = a s + k v
//   LA_MEMORY    s = a s + k (w v)        o = sum over rows of q s
// --------------------------------------------------------------------------
template <int NQ, int MODE, int PF>
__global__ __launch_bounds__(LA_WAVES * TK_WAVE) void linear_attention_kernel(LaArgs a, int dkp, const float* __restrict__ rec,
                                                                          const float2* __restrict__ gates, float* __restrict__ o) {
  const int H = a.H, dk = a.dk, columns = la_columns<MODE>(a.dv), ld_rec = la_rec_width<MODE>(H, dkp, a.dv);
  const int h = blockIdx.x, r = blockIdx.y;
  const int lane = threadIdx.x % LA_LANES, grp = threadIdx.x / LA_LANES;  // grp: a column of the workgroup's block
  const int col = blockIdx.z * (blockDim.x / LA_LANES) + grp;
  if ((col / LA_COLS) * LA_COLS >= columns) return;  // a wavefront none of whose columns exists
  const bool live = col < columns;
  const int first = a.q_start[r], last = a.q_start[r + 1];
  if (first >= last) return;
  float* s_col = a.state + (size_t)a.slots[r] * a.state_stride + ((size_t)h * columns + (live ? col : 0)) * dk;
  const bool vec = (dk % 4 == 0) && (a.state_stride % 4 == 0);
  float s[NQ][4];
#pragma unroll
  for (int n = 0; n < NQ; ++n) {
    const int i = 4 * (lane + LA_LANES * n);
    if (vec && live && i < dk) {
      const float4 v = *(const float4*)(s_col + i);
      s[n][0] = v.x; s[n][1] = v.y; s[n][2] = v.z; s[n][3] = v.w;
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e) s[n][e] = (live && i + e < dk) ? s_col[i + e] : 0.f;
    }
  }
  const float a_head = MODE == LA_CONSTANT ? a.decay[h] : 0.f;
  const int q_at = h * dkp + 4 * lane, k_at = H * dkp + q_at, v_at = la_value_at<MODE>(H, dkp) + h * columns + (live ? col : 0);

  constexpr bool CHANNEL = MODE == LA_CHANNEL, MEMORY = MODE == LA_MEMORY;
  float4 q[2][PF][NQ], k[2][PF][NQ], d[CHANNEL ? 2 : 1][CHANNEL ? PF : 1][CHANNEL ? NQ : 1];
  float v[2][PF];
  float2 g[MEMORY ? 2 : 1][MEMORY ? PF : 1];
  // rows of tokens t0 .. t0 + PF - 1 (those beyond the request's end repeat its last token and are not used)
#define LA_LOAD(B, T0)                                                               \
  _Pragma("unroll") for (int j = 0; j < PF; ++j) {                                   \
    const size_t tok = min((T0) + j, last - 1);                                      \
    const float* row = rec + tok * ld_rec;                                           \
    _Pragma("unroll") for (int n = 0; n < NQ; ++n) {                                 \
      q[B][j][n] = *(const float4*)(row + q_at + 4 * LA_LANES * n);                  \
      k[B][j][n] = *(const float4*)(row + k_at + 4 * LA_LANES * n);                  \
      if constexpr (CHANNEL) d[B][j][n] = *(const float4*)(row + H * dkp + k_at + 4 * LA_LANES * n); \
    }                                                                                \
    v[B][j] = row[v_at];                                                             \
    if constexpr (MEMORY) g[B][j] = gates[tok * H + h];                              \
  }
#define LA_STEP(B, T0)                                                               \
  _Pragma("unroll") for (int j = 0; j < PF; ++j) {                                   \
    if ((T0) + j < last) {                                                           \
      float vv = v[B][j], keep = a_head;                                             \
      if constexpr (MEMORY) {                                                        \
        keep = g[B][j].x;                                                            \
        vv *= g[B][j].y;                                                             \
      }                                                                              \
      float acc0 = 0.f, acc1 = 0.f;                                                  \
      _Pragma("unroll") for (int n = 0; n < NQ; ++n) {                               \
        const float qq[4] = {q[B][j][n].x, q[B][j][n].y, q[B][j][n].z, q[B][j][n].w}; \
        const float kk[4] = {k[B][j][n].x, k[B][j][n].y, k[B][j][n].z, k[B][j][n].w}; \
        if constexpr (CHANNEL) {                                                     \
          const float dd[4] = {d[B][j][n].x, d[B][j][n].y, d[B][j][n].z, d[B][j][n].w}; \
          _Pragma("unroll") for (int e = 0; e < 4; ++e) s[n][e] = fmaf(dd[e], s[n][e], kk[e] * vv); \
        } else {                                                                     \
          _Pragma("unroll") for (int e = 0; e < 4; ++e) {                            \
            if (MODE == LA_FORGET) s[n][e] = fmaf(kk[e], s[n][e] - vv, vv);          \
            else s[n][e] = fmaf(keep, s[n][e], kk[e] * vv);                          \
          }                                                                          \
        }                                                                            \
        acc0 = fmaf(qq[0], s[n][0], acc0); acc1 = fmaf(qq[1], s[n][1], acc1);        \
        acc0 = fmaf(qq[2], s[n][2], acc0); acc1 = fmaf(qq[3], s[n][3], acc1);        \
      }                                                                              \
      const float sum = row_sum16(acc0 + acc1);                                      \
      if (live && lane == 0) o[((size_t)((T0) + j) * H + h) * a.o_head + col] = sum; \
    }                                                                                \
  }
  LA_LOAD(0, first);
#pragma unroll 1
  for (int t0 = first; t0 < last; t0 += 2 * PF) {
    LA_LOAD(1, t0 + PF);
    LA_STEP(0, t0);
    LA_LOAD(0, t0 + 2 * PF);
    LA_STEP(1, t0 + PF);
  }
#undef LA_LOAD
#undef LA_STEP
#pragma unroll
  for (int n = 0; n < NQ; ++n) {
    const int i = 4 * (lane + LA_LANES * n);
    if (!live) continue;
    if (vec && i < dk) {
      *(float4*)(s_col + i) = make_float4(s[n][0], s[n][1], s[n][2], s[n][3]);
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (i + e < dk) s_col[i + e] = s[n][e];
    }
  }
}

// 16-byte pieces of a head's keys that a lane holds: one of the kernel's instances (1, 2, 3, 4, 6, 8); a head's keys
// are padded to 64 times that in `rec`.
static int la_pieces(int dk) {
  const int nq = (dk + 63) / 64;
  return nq <= 4 ? nq : (nq <= 6 ? 6 : 8);
}

// --------------------------------------------------------------------------
// The same for steps in which every request brings one token: the activations are computed by the lanes that need
// them (there is no pass in front and no `rec`), with the functions of the pass above, so the sums are the same bits (up to
// the order of LA_CHANNEL's low-rank sums: a workgroup computes its head's decays into LDS).  LA_MEMORY: every lane computes its head's two gates.
// --------------------------------------------------------------------------
template <int NQ, int MODE>
__global__ __launch_bounds__(LA_WAVES * TK_WAVE) void linear_attention_single_kernel(LaArgs a, const float* __restrict__ proj,
                                                                                 float* __restrict__ o) {
  constexpr int PARTS = 4;  // the low-rank sums of a channel are cut among so many threads where the workgroup has them
  __shared__ __align__(16) float decays[MODE == LA_CHANNEL ? NQ * 64 : 4], part[MODE == LA_CHANNEL ? PARTS * NQ * 64 : 4];
  const int h = blockIdx.x, r = blockIdx.y;
  const int lane = threadIdx.x % LA_LANES, grp = threadIdx.x / LA_LANES;
  const int dk = a.dk, columns = la_columns<MODE>(a.dv);
  const int col = blockIdx.z * (blockDim.x / LA_LANES) + grp;
  const bool live = col < columns;
  const int t = a.q_start[r];
  if (a.q_start[r + 1] <= t) return;
  if (MODE != LA_CHANNEL && (col / LA_COLS) * LA_COLS >= columns) return;
  float* slot = a.state + (size_t)a.slots[r] * a.state_stride;
  float* s_col = slot + ((size_t)h * columns + (live ? col : 0)) * dk;
  const bool vec = (dk % 4 == 0) && (a.state_stride % 4 == 0);
  const float* row = proj + (size_t)t * a.ld;
  float s[NQ][4];
#pragma unroll
  for (int n = 0; n < NQ; ++n) {
    const int i = 4 * (lane + LA_LANES * n);
    if (vec && live && i < dk) {
      const float4 v = *(const float4*)(s_col + i);
      s[n][0] = v.x; s[n][1] = v.y; s[n][2] = v.z; s[n][3] = v.w;
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e) s[n][e] = (live && i + e < dk) ? s_col[i + e] : 0.f;
    }
  }
  if (MODE == LA_CHANNEL) {
    const int parts = min(PARTS, max(1, (int)blockDim.x / (NQ * 64))), width = a.H * dk;
    for (int x = threadIdx.x; x < parts * NQ * 64; x += blockDim.x) {
      const int i = x % (NQ * 64);
      float z = 0.f;
      if (i < dk) {
#pragma unroll 8
        for (int r = x / (NQ * 64); r < a.rank; r += parts) z = fmaf(row[a.low_off + r], a.low_up[(size_t)r * width + h * dk + i], z);
      }
      part[x] = z;
    }
    __syncthreads();
    for (int i = threadIdx.x; i < NQ * 64; i += blockDim.x) {
      float z = 0.f;
      for (int k = 0; k < parts; ++k) z += part[k * NQ * 64 + i];
      decays[i] = i < dk ? la_channel_decay(z + a.low_bias[h * dk + i], a.tau) : 0.f;
    }
    __syncthreads();
  }
  float keep = MODE == LA_CONSTANT ? a.decay[h] : 0.f;
  float vv;
  if (MODE == LA_MEMORY) {
    const int pos = a.positions[t];
    const float gi = la_soft_cap(row[a.i_off + h] + a.i_bias[h], a.cap);
    const float gf = la_log_sigmoid(la_soft_cap(row[a.f_off + h] + a.f_bias[h], a.cap));
    const float m_prev = pos > 0 ? slot[la_max_at(a, pos - 1, h)] : 0.f;
    const float m = fmaxf(m_prev + gf, gi);
    keep = expf(gf + m_prev - m);
    vv = (live && col < a.dv ? row[a.v_off + h * a.dv + col] : 1.f) * expf(gi - m);
    if (col == a.dv && lane == 0) {
      slot[la_max_at(a, pos, h)] = m;
      a.floor[(size_t)t * a.H + h] = expf(-m);
    }
  } else {
    const float raw_v = row[a.v_off + h * a.dv + (live ? col : 0)];
    vv = MODE == LA_CONSTANT ? la_silu(raw_v) : raw_v;
  }
  float acc0 = 0.f, acc1 = 0.f;
#pragma unroll
  for (int n = 0; n < NQ; ++n) {
    const int i = 4 * (lane + LA_LANES * n);
    float qq[4], kk[4];
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const bool in = i + e < dk;
      const int c = h * dk + (in ? i + e : 0);
      if (MODE == LA_CHANNEL || MODE == LA_MEMORY) {
        qq[e] = in ? row[a.q_off + c] * a.q_scale : 0.f;
        kk[e] = in ? row[a.k_off + c] : 0.f;
      } else {
        qq[e] = in ? la_silu(row[a.q_off + c]) : 0.f;
        if (MODE == LA_CONSTANT) kk[e] = in ? la_silu(row[a.k_off + c]) : 0.f;
        else kk[e] = in ? la_forget(row[a.k_off + c], a.forget_bias[c], a.forget_low[c]) : 0.f;
      }
    }
    if (MODE == LA_CHANNEL) {
      const float4 d = *(const float4*)(decays + i);
      const float dd[4] = {d.x, d.y, d.z, d.w};
#pragma unroll
      for (int e = 0; e < 4; ++e) s[n][e] = fmaf(dd[e], s[n][e], kk[e] * vv);
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        if (MODE == LA_FORGET) s[n][e] = fmaf(kk[e], s[n][e] - vv, vv);
        else s[n][e] = fmaf(keep, s[n][e], kk[e] * vv);
      }
    }
    acc0 = fmaf(qq[0], s[n][0], acc0); acc1 = fmaf(qq[1], s[n][1], acc1);
    acc0 = fmaf(qq[2], s[n][2], acc0); acc1 = fmaf(qq[3], s[n][3], acc1);
  }
  const float sum = row_sum16(acc0 + acc1);
  if (!live) return;
  if (lane == 0) o[((size_t)t * a.H + h) * a.o_head + col] = sum;
#pragma unroll
  for (int n = 0; n < NQ; ++n) {
    const int i = 4 * (lane + LA_LANES * n);
    if (vec && i < dk) {
      *(float4*)(s_col + i) = make_float4(s[n][0], s[n][1], s[n][2], s[n][3]);
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (i + e < dk) s_col[i + e] = s[n][e];
    }
  }
}

// 32-bit words a request's slot holds for these sizes.
TK_API int tk_linear_attention_state_words(int mode, int H, int dk, int dv) {
  return mode == LA_MEMORY ? (H * (dv + 1) * dk + 2 * H + 3) / 4 * 4 : H * dv * dk;
}
// 32-bit words of working memory a token of a step with these sizes and this longest portion takes.
TK_API int tk_linear_attention_work_words(int mode, int H, int dk, int dv, int longest) {
  if (longest <= 1) return 0;
  const int dkp = la_pieces(dk) * 64;
  if (mode == LA_MEMORY) return la_rec_width<LA_MEMORY>(H, dkp, dv) + 2 * H;
  return mode == LA_CHANNEL ? la_rec_width<LA_CHANNEL>(H, dkp, dv) : la_rec_width<LA_CONSTANT>(H, dkp, dv);
}

void la_launch_gates(const LaArgs& a, float2* gates, int log_decay, hipStream_t stream) {
  hipLaunchKernelGGL(linear_attention_gates_kernel, dim3(a.H, a.n_requests), dim3(LA_GATES), 0, stream, a, gates, log_decay);
}

template <int MODE>
static int la_run(const LaArgs& a, hipStream_t stream) {
  const int columns = la_columns<MODE>(a.dv), all_waves = (columns + LA_COLS - 1) / LA_COLS;
  const int nq = la_pieces(a.dk), dkp = 64 * nq;
  if (a.longest <= 1) {
    const int waves = min(LA_WAVES, all_waves);
    const dim3 grid(a.H, a.n_requests, (all_waves + waves - 1) / waves), block(waves * TK_WAVE);
#define LA_SINGLE(NQ) hipLaunchKernelGGL((linear_attention_single_kernel<NQ, MODE>), grid, block, 0, stream, a, a.proj, a.o)
    if (nq <= 1) LA_SINGLE(1);
    else if (nq <= 2) LA_SINGLE(2);
    else if (nq <= 3) LA_SINGLE(3);
    else if (nq <= 4) LA_SINGLE(4);
    else if (nq <= 6) LA_SINGLE(6);
    else LA_SINGLE(8);
#undef LA_SINGLE
    TK_CHECK_LAUNCH("linear_attention");
    return 0;
  }
  const int ld_rec = la_rec_width<MODE>(a.H, dkp, a.dv);
  const dim3 pgrid((ld_rec + 255) / 256, a.n_tokens);
  hipLaunchKernelGGL(linear_attention_prepare_kernel<MODE>, pgrid, dim3(256), 0, stream, a, dkp);
  float2* gates = nullptr;
  if (MODE == LA_CHANNEL)
    hipLaunchKernelGGL(linear_attention_decay_kernel, dim3((a.H * dkp + 255) / 256, (a.n_tokens + LA_TOKENS - 1) / LA_TOKENS), dim3(256),
                       0, stream, a, dkp);
  if (MODE == LA_MEMORY) {
    gates = (float2*)(a.rec + (size_t)a.n_tokens * ld_rec);  // (rows are multiples of 16 bytes)
    la_launch_gates(a, gates, 0, stream);
  }
  // A long walk is a chain of arithmetic in every wavefront: one wavefront a workgroup then spreads a prompt's few
  // wavefronts over all compute units (measured: 2 048 tokens of 8 heads of 128 x 128 in 180 us, against 360 us with
  // eight wavefronts a workgroup).  Steps of few tokens a request launch thousands of short wavefronts, in workgroups of eight.
  const int waves = a.longest > 16 ? 1 : min(LA_WAVES, all_waves);
  const dim3 grid(a.H, a.n_requests, (all_waves + waves - 1) / waves), block(waves * TK_WAVE);
#define LA_CASE(NQ, PF) hipLaunchKernelGGL((linear_attention_kernel<NQ, MODE, PF>), grid, block, 0, stream, a, dkp, a.rec, gates, a.o)
  if (nq <= 1) LA_CASE(1, 4);
  else if (nq <= 2) LA_CASE(2, 4);
  else if (nq <= 3) LA_CASE(3, 2);
  else if (nq <= 4) LA_CASE(4, 2);
  else if (nq <= 6) LA_CASE(6, 1);
  else LA_CASE(8, 1);
#undef LA_CASE
  TK_CHECK_LAUNCH("linear_attention");
  return 0;
}

TK_API int tk_linear_attention(int mode, const LaArgs* args, hipStream_t stream) {
  const LaArgs& a = *args;
  TK_REQUIRE(a.n_tokens >= 0 && a.n_requests >= 0 && a.H > 0 && a.dk > 0 && a.dv > 0 && a.dk <= 512,
             "linear_attention: bad sizes tokens=%d requests=%d heads=%d dk=%d dv=%d (dk up to 512)", a.n_tokens, a.n_requests, a.H,
             a.dk, a.dv);
  TK_REQUIRE(mode >= LA_CONSTANT && mode <= LA_MEMORY, "linear_attention: no form %d", mode);
  TK_REQUIRE(mode != LA_CONSTANT || a.decay, "linear_attention: the constant form needs a decay a head");
  TK_REQUIRE(mode != LA_FORGET || (a.forget_bias && a.forget_low), "linear_attention: the forget-gate form needs a bias and a lower bound");
  TK_REQUIRE(mode != LA_CHANNEL || (a.low_up && a.low_bias && a.rank > 0 && a.low_off >= 0 && a.low_off + a.rank <= a.ld && a.tau > 0.f),
             "linear_attention: the decay-a-channel form needs its low-rank projection's second matrix, a bias and a positive tau");
  TK_REQUIRE(mode != LA_MEMORY || (a.i_bias && a.f_bias && a.floor && a.positions && a.cap > 0.f && a.i_off >= 0 && a.f_off >= 0 &&
                                   a.i_off + a.H <= a.ld && a.f_off + a.H <= a.ld),
             "linear_attention: the matrix-memory form needs its gates' sums and biases, the positions and a positive cap");
  const bool single = a.longest <= 1;
  TK_REQUIRE(a.q_off >= 0 && a.k_off >= 0 && a.v_off >= 0 && a.q_off + a.H * a.dk <= a.ld && a.k_off + a.H * a.dk <= a.ld &&
                 a.v_off + a.H * a.dv <= a.ld, "linear_attention: a part lies outside the rows");
  TK_REQUIRE(a.proj && a.state && a.q_start && a.slots && a.o && (a.rec || single) && a.n_requests < 65536 && a.n_tokens < 65536 &&
                 a.state_stride >= (size_t)tk_linear_attention_state_words(mode, a.H, a.dk, a.dv) &&
                 a.o_head >= a.dv + (mode == LA_MEMORY ? 1 : 0),
             "linear_attention: a pointer is missing, the state's or the result's rows are too short or the step too large");
  TK_REQUIRE((((uintptr_t)a.rec | (uintptr_t)a.state) & 15) == 0, "linear_attention: rec and state must start at multiples of 16 bytes");
  TK_REQUIRE(a.longest >= 1, "linear_attention: the longest portion of a step with tokens is at least one token");
  TK_REQUIRE(a.n_chunks == 0 || (a.n_chunks > 0 && a.chunk_req && a.chunk_row0 && a.first_chunk && la_chunks_take(mode, a.dk, a.longest)),
             "linear_attention: the chunked form does not take these sizes, or its plan is missing");
  if (a.n_requests == 0 || a.n_tokens == 0) return 0;
  if (a.n_chunks > 0) return la_run_chunks(mode, a, stream);
  switch (mode) {
    case LA_CONSTANT: return la_run<LA_CONSTANT>(a, stream);
    case LA_FORGET: return la_run<LA_FORGET>(a, stream);
    case LA_CHANNEL: return la_run<LA_CHANNEL>(a, stream);
    default: return la_run<LA_MEMORY>(a, stream);
  }
}

// --------------------------------------------------------------------------
// Behind the recurrence: every group's `size` numbers of a token divided by their root mean square, times a
// weight (one of `size` numbers that the groups share, or, `w_all`, a number for every element of a row), times
// sigmoid(gate) or (`silu_gate`) silu(gate) where there is a gate, times `scale`; rounded once
// to T.  A group is a head (a norm head by head) or the whole row (groups = 1); a group's numbers begin `o_group` apart.
// `floor` (null or a number a group): the group's numbers are first divided by max(|d|, floor) + 1e-6 with d the number
// behind the last of them.  A wavefront a (token, group).
// --------------------------------------------------------------------------
struct GroupNormArgs {
  const float* o;
  int o_group;
  const float* gate;
  int ld_gate, silu_gate, groups;
  const float* w;
  int w_all;
  const float* floor;
  float eps, scale;
  int ld_out, size;
};
#define GN_FLOOR_EPS 1e-6f
__device__ __forceinline__ float gn_divisor(const GroupNormArgs& a, const float* x, long unit) {
  return a.floor ? 1.0f / (fmaxf(fabsf(x[a.size]), a.floor[unit]) + GN_FLOOR_EPS) : 1.f;
}
__device__ __forceinline__ float gn_gate(const GroupNormArgs& a, float y, float g) { return y * (a.silu_gate ? la_silu(g) : la_sigmoid(g)); }

template <typename T>
__global__ __launch_bounds__(256) void group_norm_gate_kernel(GroupNormArgs a, T* __restrict__ out, long units) {
  const int lane = threadIdx.x & (TK_WAVE - 1), size = a.size;
  const long unit = (long)blockIdx.x * (blockDim.x / TK_WAVE) + threadIdx.x / TK_WAVE;
  if (unit >= units) return;
  const long t = unit / a.groups;
  const int g = (int)(unit % a.groups);
  const float* __restrict__ x = a.o + (size_t)unit * a.o_group;
  const float* __restrict__ w = a.w + (a.w_all ? (size_t)g * size : 0);
  const float div = gn_divisor(a, x, unit);
  float ss = 0.f;
  for (int i = lane; i < size; i += TK_WAVE) {
    const float v = x[i] * div;
    ss = fmaf(v, v, ss);
  }
  ss = wave_sum(ss);
  const float rstd = 1.0f / sqrtf(ss / (float)size + a.eps);
  for (int i = lane; i < size; i += TK_WAVE) {
    float y = x[i] * div * rstd * w[i];
    if (a.gate) y = gn_gate(a, y, a.gate[(size_t)t * a.ld_gate + (size_t)g * size + i]);
    out[(size_t)t * a.ld_out + (size_t)g * size + i] = from_f32<T>(y * a.scale);
  }
}

// The same with a workgroup a (token, group), for groups of many numbers (one norm over all heads): a wavefront alone
// would walk such a row as a chain of loads.
template <typename T>
__global__ __launch_bounds__(256) void group_norm_gate_wide_kernel(GroupNormArgs a, T* __restrict__ out) {
  __shared__ float red[16];
  const int size = a.size;
  const long unit = blockIdx.x;
  const long t = unit / a.groups;
  const int g = (int)(unit % a.groups);
  const float* __restrict__ x = a.o + (size_t)unit * a.o_group;
  const float* __restrict__ w = a.w + (a.w_all ? (size_t)g * size : 0);
  const float* __restrict__ gate = a.gate ? a.gate + (size_t)t * a.ld_gate + (size_t)g * size : nullptr;
  T* __restrict__ dst = out + (size_t)t * a.ld_out + (size_t)g * size;
  const float div = gn_divisor(a, x, unit);
  float ss = 0.f;
  if (size % 4 == 0 && size <= 4 * 256 * 4 && ((uintptr_t)x & 15) == 0) {
    // the row in registers: up to four 16-byte pieces a thread, asked for together
    float4 v[4];
#pragma unroll
    for (int q = 0; q < 4; ++q) {
      const int i = threadIdx.x + q * 256;
      v[q] = i < size / 4 ? ((const float4*)x)[i] : make_float4(0.f, 0.f, 0.f, 0.f);
      v[q].x *= div; v[q].y *= div; v[q].z *= div; v[q].w *= div;
      ss = fmaf(v[q].x, v[q].x, ss); ss = fmaf(v[q].y, v[q].y, ss); ss = fmaf(v[q].z, v[q].z, ss); ss = fmaf(v[q].w, v[q].w, ss);
    }
    ss = block_sum(ss, red);
    const float rstd = 1.0f / sqrtf(ss / (float)size + a.eps);
#pragma unroll
    for (int q = 0; q < 4; ++q) {
      const int i = threadIdx.x + q * 256;
      if (i < size / 4) {
        const float xs[4] = {v[q].x, v[q].y, v[q].z, v[q].w};
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const int c = 4 * i + e;
          float y = xs[e] * rstd * w[c];
          if (gate) y = gn_gate(a, y, gate[c]);
          dst[c] = from_f32<T>(y * a.scale);
        }
      }
    }
    return;
  }
  for (int i = threadIdx.x; i < size; i += blockDim.x) {
    const float v = x[i] * div;
    ss = fmaf(v, v, ss);
  }
  ss = block_sum(ss, red);
  const float rstd = 1.0f / sqrtf(ss / (float)size + a.eps);
  for (int i = threadIdx.x; i < size; i += blockDim.x) {
    float y = x[i] * div * rstd * w[i];
    if (gate) y = gn_gate(a, y, gate[i]);
    dst[i] = from_f32<T>(y * a.scale);
  }
}

TK_API int tk_group_norm_gate(int dt, const float* o, int o_group, const float* gate, int ld_gate, int silu_gate, const float* w, int w_all,
                              const float* floor, float eps, float scale, void* out, int ld_out, int n_tokens, int groups, int size,
                              hipStream_t stream) {
  TK_REQUIRE(n_tokens >= 0 && groups > 0 && size > 0 && o && w && out, "group_norm_gate: bad sizes %d %d %d or a pointer is missing",
             n_tokens, groups, size);
  TK_REQUIRE(ld_out >= groups * size && (!gate || ld_gate >= groups * size) && o_group >= size + (floor ? 1 : 0),
             "group_norm_gate: a row stride is too short");
  if (n_tokens == 0) return 0;
  const long units = (long)n_tokens * groups;
  const long blocks = (units + 3) / 4;
  TK_REQUIRE(units < (1l << 31), "group_norm_gate: too many rows");
  const GroupNormArgs a{o, o_group, gate, ld_gate, silu_gate, groups, w, w_all, floor, eps, scale, ld_out, size};
  if (size > 256) {
    if (dt == TK_F32)
      hipLaunchKernelGGL(group_norm_gate_wide_kernel<float>, dim3((unsigned)units), dim3(256), 0, stream, a, (float*)out);
    else
      hipLaunchKernelGGL(group_norm_gate_wide_kernel<bf16_t>, dim3((unsigned)units), dim3(256), 0, stream, a, (bf16_t*)out);
  } else {
    if (dt == TK_F32)
      hipLaunchKernelGGL(group_norm_gate_kernel<float>, dim3((unsigned)blocks), dim3(256), 0, stream, a, (float*)out, units);
    else
      hipLaunchKernelGGL(group_norm_gate_kernel<bf16_t>, dim3((unsigned)blocks), dim3(256), 0, stream, a, (bf16_t*)out, units);
  }
  TK_CHECK_LAUNCH("group_norm_gate");
  return 0;
}

// --------------------------------------------------------------------------
// out[t, i] = x[t, i] * sigmoid(gate[t, i]) * scale, element by element (rows a stride apart), 32-bit arithmetic,
// one rounding.
// --------------------------------------------------------------------------
template <typename T>
__global__ void sigmoid_gate_kernel(const T* __restrict__ x, int ld_x, const T* __restrict__ gate, int ld_gate, float scale,
                                    T* __restrict__ out, int ld_out, int width) {
  const int i = blockIdx.x * blockDim.x + threadIdx.x;
  const size_t t = blockIdx.y;
  if (i < width)
    out[t * ld_out + i] = from_f32<T>(to_f32<T>(x[t * ld_x + i]) * la_sigmoid(to_f32<T>(gate[t * ld_gate + i])) * scale);
}

// (16 bytes a load where widths, strides and addresses allow)
template <typename T>
__global__ void sigmoid_gate_vec_kernel(const T* __restrict__ x, int ld_x, const T* __restrict__ gate, int ld_gate, float scale,
                                        T* __restrict__ out, int ld_out, int width) {
  constexpr int N = 16 / sizeof(T);
  union Piece { uint4 raw; T v[N]; };
  const int i = (blockIdx.x * blockDim.x + threadIdx.x) * N;
  const size_t t = blockIdx.y;
  if (i >= width) return;
  Piece a, g, o;
  a.raw = *(const uint4*)(x + t * ld_x + i);
  g.raw = *(const uint4*)(gate + t * ld_gate + i);
#pragma unroll
  for (int e = 0; e < N; ++e) o.v[e] = from_f32<T>(to_f32<T>(a.v[e]) * la_sigmoid(to_f32<T>(g.v[e])) * scale);
  *(uint4*)(out + t * ld_out + i) = o.raw;
}

TK_API int tk_sigmoid_gate(int dt, const void* x, int ld_x, const void* gate, int ld_gate, float scale, void* out, int ld_out,
                           int rows, int width, hipStream_t stream) {
  TK_REQUIRE(rows >= 0 && rows < 65536 && width > 0 && x && gate && out && ld_x >= width && ld_gate >= width && ld_out >= width,
             "sigmoid_gate: bad sizes %d %d, a pointer is missing or a stride is too short", rows, width);
  if (rows == 0) return 0;
  const dim3 grid((width + 255) / 256, rows);
  const int per = dt == TK_F32 ? 4 : 8;
  if (width % per == 0 && ld_x % per == 0 && ld_gate % per == 0 && ld_out % per == 0 &&
      (((uintptr_t)x | (uintptr_t)gate | (uintptr_t)out) & 15) == 0) {
    const dim3 vgrid((width / per + 127) / 128, rows);
    if (dt == TK_F32)
      hipLaunchKernelGGL(sigmoid_gate_vec_kernel<float>, vgrid, dim3(128), 0, stream, (const float*)x, ld_x, (const float*)gate,
                         ld_gate, scale, (float*)out, ld_out, width);
    else
      hipLaunchKernelGGL(sigmoid_gate_vec_kernel<bf16_t>, vgrid, dim3(128), 0, stream, (const bf16_t*)x, ld_x, (const bf16_t*)gate,
                         ld_gate, scale, (bf16_t*)out, ld_out, width);
    TK_CHECK_LAUNCH("sigmoid_gate");
    return 0;
  }
  if (dt == TK_F32)
    hipLaunchKernelGGL(sigmoid_gate_kernel<float>, grid, dim3(256), 0, stream, (const float*)x, ld_x, (const float*)gate, ld_gate,
                       scale, (float*)out, ld_out, width);
  else
    hipLaunchKernelGGL(sigmoid_gate_kernel<bf16_t>, grid, dim3(256), 0, stream, (const bf16_t*)x, ld_x, (const bf16_t*)gate, ld_gate,
                       scale, (bf16_t*)out, ld_out, width);
  TK_CHECK_LAUNCH("sigmoid_gate");
  return 0;
}

// --------------------------------------------------------------------------
// A short causal convolution over time on every channel, added to its input:
//     out_t = h_t + sum_j w[j][c] * h_(t - taps + 1 + j)      (zeros before a request's first token)
// The taps are kept tap by tap, w [taps][width], so that neighbouring channels' weights of one tap lie together.
// The last taps - 1 inputs of a request live in its slot's `tail` [taps - 1][width] (32-bit, oldest first,
// zeros when the request takes the slot).  A thread a (token, channel).  FUSE_TAIL (every request of the step
// brings one token): the thread also moves its channel's tail on, which it alone reads; else the tail kernel
// below runs afterwards.
// --------------------------------------------------------------------------
#define SC_MAX_TAPS 16
template <typename T, bool FUSE_TAIL>
__global__ void short_conv_kernel(const T* __restrict__ h, int ld, const float* __restrict__ w, int taps, float* __restrict__ tails,
                                  size_t tail_stride, const int* __restrict__ q_start, const int* __restrict__ token_req,
                                  const int* __restrict__ slots, T* __restrict__ out, int width) {
  const int t = blockIdx.y;
  const int c = blockIdx.x * blockDim.x + threadIdx.x;
  if (c >= width) return;
  const int r = token_req[t];
  const int first = q_start[r];
  const int local = t - first;
  float* tail = tails + (size_t)slots[r] * tail_stride;
  float acc = 0.f, cur = 0.f;
  for (int j = 0; j < taps; ++j) {
    const int src = local - (taps - 1) + j;
    const float x = src >= 0 ? to_f32<T>(h[(size_t)(first + src) * ld + c]) : tail[(size_t)(src + taps - 1) * width + c];
    acc = fmaf(w[(size_t)j * width + c], x, acc);
    cur = x;
    if (FUSE_TAIL && j >= 1) tail[(size_t)(j - 1) * width + c] = x;  // (local is 0: entry j - 1 was read a tap ago)
  }
  out[(size_t)t * width + c] = from_f32<T>(cur + acc);
}

// The same with 16 bytes a load: a thread 16 / sizeof(T) neighbouring channels (widths and strides that are multiples
// of that, rows that start at multiples of 16 bytes).
template <typename T, bool FUSE_TAIL>
__global__ void short_conv_vec_kernel(const T* __restrict__ h, int ld, const float* __restrict__ w, int taps, float* __restrict__ tails,
                                      size_t tail_stride, const int* __restrict__ q_start, const int* __restrict__ token_req,
                                      const int* __restrict__ slots, T* __restrict__ out, int width) {
  constexpr int N = 16 / sizeof(T);
  union Piece { uint4 raw; T v[N]; };
  const int t = blockIdx.y;
  const int c0 = (blockIdx.x * blockDim.x + threadIdx.x) * N;
  if (c0 >= width) return;
  const int r = token_req[t];
  const int first = q_start[r];
  const int local = t - first;
  float* tail = tails + (size_t)slots[r] * tail_stride;
  float acc[N], cur[N];
#pragma unroll
  for (int e = 0; e < N; ++e) acc[e] = cur[e] = 0.f;
#pragma unroll 4
  for (int j = 0; j < taps; ++j) {
    const int src = local - (taps - 1) + j;
    float x[N];
    if (src >= 0) {
      Piece p;
      p.raw = *(const uint4*)(h + (size_t)(first + src) * ld + c0);
#pragma unroll
      for (int e = 0; e < N; ++e) x[e] = to_f32<T>(p.v[e]);
    } else {
      const float4* from = (const float4*)(tail + (size_t)(src + taps - 1) * width + c0);
#pragma unroll
      for (int e = 0; e < N; e += 4) {
        const float4 v = from[e / 4];
        x[e] = v.x; x[e + 1] = v.y; x[e + 2] = v.z; x[e + 3] = v.w;
      }
    }
    const float4* wj = (const float4*)(w + (size_t)j * width + c0);
#pragma unroll
    for (int e = 0; e < N; e += 4) {
      const float4 g = wj[e / 4];
      acc[e] = fmaf(g.x, x[e], acc[e]); acc[e + 1] = fmaf(g.y, x[e + 1], acc[e + 1]);
      acc[e + 2] = fmaf(g.z, x[e + 2], acc[e + 2]); acc[e + 3] = fmaf(g.w, x[e + 3], acc[e + 3]);
    }
#pragma unroll
    for (int e = 0; e < N; ++e) cur[e] = x[e];
    if (FUSE_TAIL && j >= 1) {  // (local is 0: entry j - 1 was read a tap ago)
      float4* to = (float4*)(tail + (size_t)(j - 1) * width + c0);
#pragma unroll
      for (int e = 0; e < N; e += 4) to[e / 4] = make_float4(x[e], x[e + 1], x[e + 2], x[e + 3]);
    }
  }
  Piece o;
#pragma unroll
  for (int e = 0; e < N; ++e) o.v[e] = from_f32<T>(cur[e] + acc[e]);
  *(uint4*)(out + (size_t)t * width + c0) = o.raw;
}

// The tails after the step: the last taps - 1 inputs of every request, from this step's rows and, where the
// step brought fewer, from the old tail.  A thread a (request, channel); it reads all it needs before it writes.
template <typename T>
__global__ void short_conv_tail_kernel(const T* __restrict__ h, int ld, int taps, float* __restrict__ tails, size_t tail_stride,
                                       const int* __restrict__ q_start, const int* __restrict__ slots, int width) {
  const int r = blockIdx.y;
  const int c = blockIdx.x * blockDim.x + threadIdx.x;
  if (c >= width) return;
  const int first = q_start[r], n = q_start[r + 1] - first;
  float* tail = tails + (size_t)slots[r] * tail_stride;
  float keep[SC_MAX_TAPS];
#pragma unroll
  for (int s = 0; s < SC_MAX_TAPS - 1; ++s) {
    if (s < taps - 1) {
      const int src = n - (taps - 1) + s;
      keep[s] = src >= 0 ? to_f32<T>(h[(size_t)(first + src) * ld + c]) : tail[(size_t)(src + taps - 1) * width + c];
    }
  }
#pragma unroll
  for (int s = 0; s < SC_MAX_TAPS - 1; ++s)
    if (s < taps - 1) tail[(size_t)s * width + c] = keep[s];
}

TK_API int tk_short_conv(int dt, const void* h, int ld, const float* w, int taps, float* tails, size_t tail_stride,
                         const int* q_start, const int* token_req, const int* slots, void* out, int n_tokens, int n_requests,
                         int width, int single_tokens, hipStream_t stream) {
  TK_REQUIRE(n_tokens >= 0 && n_requests >= 0 && width > 0 && taps >= 1 && taps <= SC_MAX_TAPS && ld >= width,
             "short_conv: bad sizes tokens=%d requests=%d width=%d taps=%d", n_tokens, n_requests, width, taps);
  TK_REQUIRE(h && w && out && q_start && token_req && slots && (taps == 1 || (tails && tail_stride >= (size_t)(taps - 1) * width)),
             "short_conv: a pointer is missing or the tails' rows are too short");
  TK_REQUIRE(n_tokens < 65536 * 32 && n_requests < 65536, "short_conv: too many rows for one call");
  if (n_tokens == 0) return 0;
  TK_REQUIRE(n_tokens < 65536, "short_conv: %d tokens are too many for one call", n_tokens);
  const dim3 grid((width + 255) / 256, n_tokens), tail_grid((width + 255) / 256, n_requests);
  const int per = dt == TK_F32 ? 4 : 8;  // channels of 16 bytes
  const bool vec = width % per == 0 && ld % per == 0 && (((uintptr_t)h | (uintptr_t)out | (uintptr_t)w) & 15) == 0 &&
                   (taps == 1 || ((((uintptr_t)tails) & 15) == 0 && tail_stride % 4 == 0));
  const dim3 vgrid((width / per + 127) / 128, n_tokens);
#define SC_VEC(T)                                                                                                                    \
  do {                                                                                                                               \
    if (single_tokens)                                                                                                               \
      hipLaunchKernelGGL((short_conv_vec_kernel<T, true>), vgrid, dim3(128), 0, stream, (const T*)h, ld, w, taps, tails, tail_stride, \
                         q_start, token_req, slots, (T*)out, width);                                                                 \
    else {                                                                                                                           \
      hipLaunchKernelGGL((short_conv_vec_kernel<T, false>), vgrid, dim3(128), 0, stream, (const T*)h, ld, w, taps, tails,            \
                         tail_stride, q_start, token_req, slots, (T*)out, width);                                                    \
      if (taps > 1)                                                                                                                  \
        hipLaunchKernelGGL(short_conv_tail_kernel<T>, tail_grid, dim3(256), 0, stream, (const T*)h, ld, taps, tails, tail_stride,    \
                           q_start, slots, width);                                                                                   \
    }                                                                                                                                \
  } while (0)
  if (vec) {
    if (dt == TK_F32) SC_VEC(float);
    else SC_VEC(bf16_t);
    TK_CHECK_LAUNCH("short_conv");
    return 0;
  }
#undef SC_VEC
#define SC_CASE(T)                                                                                                                   \
  do {                                                                                                                               \
    if (single_tokens)                                                                                                               \
      hipLaunchKernelGGL((short_conv_kernel<T, true>), grid, dim3(256), 0, stream, (const T*)h, ld, w, taps, tails, tail_stride,     \
                         q_start, token_req, slots, (T*)out, width);                                                                 \
    else {                                                                                                                           \
      hipLaunchKernelGGL((short_conv_kernel<T, false>), grid, dim3(256), 0, stream, (const T*)h, ld, w, taps, tails, tail_stride,    \
                         q_start, token_req, slots, (T*)out, width);                                                                 \
      if (taps > 1)                                                                                                                  \
        hipLaunchKernelGGL(short_conv_tail_kernel<T>, tail_grid, dim3(256), 0, stream, (const T*)h, ld, taps, tails, tail_stride,    \
                           q_start, slots, width);                                                                                   \
    }                                                                                                                                \
  } while (0)
  if (dt == TK_F32) SC_CASE(float);
  else SC_CASE(bf16_t);
#undef SC_CASE
  TK_CHECK_LAUNCH("short_conv");
  return 0;
}
