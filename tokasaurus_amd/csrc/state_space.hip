// A selective state-space mixer (Mamba-2's form) as a recurrence over the tokens of each request, and the gated norm
// behind it.  Per head, with a matrix S [N][dv] kept per request in 32-bit and B, C shared by the heads of a group:
//     u = silu(conv(.)) for x | B | C       a causal convolution over time on every channel, with a bias
//     dt = softplus(. + dt_bias[h])         a = exp(-exp(A_log[h]) dt)
//     S <- a S + dt B x^T                   y = S^T C + D[h] x
// All of it is read from the 32-bit sums `proj` of one stacked product (x | B | C are `channels` neighbouring columns,
// dt another H).  Step sizes, decays, the state and everything summed into it or read out of it are 32-bit; with
// bfloat16 storage (`round`) the activated convolution's result is rounded once to bfloat16, whatever the form below.
//
// Three forms of the same sums:
//   single   every request of the step brings one token: one kernel
//   scan     token by token: portions of few tokens, and the 32-bit storage type
//   chunks   bfloat16 storage, long portions: 64 tokens at a time as products on the matrix cores
//
// What a slot keeps: [H][dv][N] the matrices (a value column's N numbers lie together), and from `ring_off` on the
// convolution's last inputs as a ring [taps][channels]: the input of position p lies in entry p % taps.  A token needs
// the entries of the taps - 1 positions before it and never the one that it writes, so workgroups that read the same
// channels need no order among themselves.  Positions in front of a request's start count as zeros.
//
// In the first two the columns of S do not meet: a column is owned by SS_LANES neighbouring lanes that cut N between them and add up
// through the wavefront's own data paths, always in the same order, so a token's result does not depend on how its
// request's tokens were cut into steps or on what shares the batch.  The chunks' products add in another order.
#include <math.h>

#include "common.h"

typedef float v4f __attribute__((ext_vector_type(4)));
typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8_t;
typedef uint32_t u32x4 __attribute__((ext_vector_type(4)));

#define SS_LANES 16
#define SS_COLS 4    // value columns a wavefront owns
#define SS_WAVES 16      // most wavefronts of a workgroup that takes one token
#define SS_SCAN_WAVES 4  // of one that walks (its rows ahead need registers)

__device__ __forceinline__ float ss_silu(float x) { return x / (1.0f + expf(-x)); }
__device__ __forceinline__ float ss_softplus(float x) { return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))); }
// the logarithm of a token's decay
__device__ __forceinline__ float ss_log_decay(float a_log, float dt) { return -__fmul_rn(expf(a_log), dt); }
__device__ __forceinline__ float ss_decay(float a_log, float dt) { return expf(ss_log_decay(a_log, dt)); }

struct SsArgs {
  const float* proj;      // [tokens][ld]
  int ld, x_off, dt_off;  // first column of x | B | C, and of dt
  const float *conv_w, *conv_b;  // [taps][channels], [channels]
  int taps, channels;
  const float *a_log, *dt_bias, *d_skip;  // [H]
  float* state;
  size_t state_stride, ring_off;
  const int *q_start, *token_req, *slots, *positions;
  float* y;  // [tokens][H * dv]
  int H, G, N, dv;
  int round;  // the activated convolution is rounded to bfloat16
};

// The activated convolution of channel c at the token of row t: `local` tokens of its request stand before it in this
// step, `pos` is its position.
__device__ __forceinline__ float ss_channel(const SsArgs& a, int t, int local, int pos, const float* ring, int c) {
  float acc = a.conv_b[c];
  for (int j = 0; j < a.taps; ++j) {
    const int back = a.taps - 1 - j;
    float v = 0.f;
    if (back <= local) v = a.proj[(size_t)(t - back) * a.ld + a.x_off + c];
    else if (back <= pos) v = ring[(size_t)((pos - back) % a.taps) * a.channels + c];
    acc = fmaf(a.conv_w[(size_t)j * a.channels + c], v, acc);
  }
  acc = ss_silu(acc);
  return a.round ? round_to<bf16_t>(acc) : acc;
}

// The same for four neighbouring channels with 16 bytes a load (the entry point has checked strides and addresses).
__device__ __forceinline__ void ss_channel4(const SsArgs& a, int t, int local, int pos, const float* ring, int c, float (&out)[4]) {
  float4 acc = *(const float4*)(a.conv_b + c);
#pragma unroll 4
  for (int j = 0; j < a.taps; ++j) {
    const int back = a.taps - 1 - j;
    float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
    if (back <= local) v = *(const float4*)(a.proj + (size_t)(t - back) * a.ld + a.x_off + c);
    else if (back <= pos) v = *(const float4*)(ring + (size_t)((pos - back) % a.taps) * a.channels + c);
    const float4 w = *(const float4*)(a.conv_w + (size_t)j * a.channels + c);
    acc.x = fmaf(w.x, v.x, acc.x); acc.y = fmaf(w.y, v.y, acc.y); acc.z = fmaf(w.z, v.z, acc.z); acc.w = fmaf(w.w, v.w, acc.w);
  }
  const float r[4] = {ss_silu(acc.x), ss_silu(acc.y), ss_silu(acc.z), ss_silu(acc.w)};
#pragma unroll
  for (int e = 0; e < 4; ++e) out[e] = a.round ? round_to<bf16_t>(r[e]) : r[e];
}

// 16-byte pieces of a column that a lane holds: one of the kernels' instances (1, 2, 3, 4, 6, 8)
static int ss_pieces(int n) {
  const int nq = (n + 63) / 64;
  return nq <= 4 ? nq : (nq <= 6 ? 6 : 8);
}
// The activated rows that the scan and the chunks read, a row a token: [x: inner | B: G x np | C: G x np] of T (32-bit for
// the scan, bfloat16 for the chunks), x padded to a multiple of 8, B and C with zeros from N on; behind all rows
// [tokens][H][2] in 32-bit: the decay (the chunks: its logarithm) and dt.  np is a whole number of a lane's pieces for the
// scan (64 each: a padded row of S meets a zero of C), of 32 for the chunks.
__host__ __device__ __forceinline__ int ss_rec_b(int inner) { return (inner + 7) / 8 * 8; }
__host__ __device__ __forceinline__ int ss_rec_width(int inner, int G, int np) { return ss_rec_b(inner) + 2 * G * np; }

// --------------------------------------------------------------------------
// In front of the scan and the chunks, once a token: convolution and activations, step sizes and decays.
// A thread V neighbouring numbers of a row (4, with 16 bytes a load, where the sizes allow; else 1).
// --------------------------------------------------------------------------
template <typename T, int V>
__global__ __launch_bounds__(256) void ss_prepare_kernel(SsArgs a, T* __restrict__ rec, int ld_rec, int np, float2* __restrict__ ev,
                                                         int log_decay) {
  const int t = blockIdx.y;
  int x = (blockIdx.x * blockDim.x + threadIdx.x) * V;
  if (x >= ld_rec) {
    x = (x - ld_rec) / V;
    if (x >= a.H) return;
    const float dt = ss_softplus(a.proj[(size_t)t * a.ld + a.dt_off + x] + a.dt_bias[x]);
    ev[(size_t)t * a.H + x] = make_float2(log_decay ? ss_log_decay(a.a_log[x], dt) : ss_decay(a.a_log[x], dt), dt);
    return;
  }
  const int inner = a.H * a.dv, b0 = ss_rec_b(inner);
  const int r = a.token_req[t];
  const int local = t - a.q_start[r];
  const float* ring = a.state + (size_t)a.slots[r] * a.state_stride + a.ring_off;
  int c = -1;  // (padding)
  if (x < b0) {
    if (x < inner) c = x;
  } else {
    const int g = (x - b0) / np, i = (x - b0) % np;  // g counts the groups of B, then those of C
    if (i < a.N) c = inner + g * a.N + i;
  }
  struct alignas(sizeof(T) * V) Piece { T v[V]; } o;
#pragma unroll
  for (int e = 0; e < V; ++e) o.v[e] = from_f32<T>(0.f);
  if (c >= 0) {
    if constexpr (V == 4) {
      float v[4];
      ss_channel4(a, t, local, a.positions[t], ring, c, v);
#pragma unroll
      for (int e = 0; e < 4; ++e) o.v[e] = from_f32<T>(v[e]);
    } else {
      o.v[0] = from_f32<T>(ss_channel(a, t, local, a.positions[t], ring, c));
    }
  }
  *(Piece*)(rec + (size_t)t * ld_rec + x) = o;
}

// The last `taps` inputs of the step's tokens into the ring (fewer when it brings fewer: the rest of the ring stays), by
// all threads of a request's workgroups together: `first_thread` of `threads`.  The pass in front has read the ring.
__device__ __forceinline__ void ss_move_ring(const SsArgs& a, float* slot, int first, int last, int first_thread, int threads) {
  if (a.taps <= 1) return;
  for (int c = first_thread; c < a.channels; c += threads)
    for (int t = max(first, last - a.taps); t < last; ++t)
      slot[a.ring_off + (size_t)(a.positions[t] % a.taps) * a.channels + c] = a.proj[(size_t)t * a.ld + a.x_off + c];
}

// --------------------------------------------------------------------------
// The scan.  A wavefront owns SS_COLS value columns of one (head, request); lane l of a
// column's SS_LANES holds rows 4 * (l + SS_LANES * n) + e, n < NQ, e < 4.  No LDS and no barrier: the wavefronts of a
// group's heads read the same rows of `rec` through the caches, two groups of PF tokens ahead of the arithmetic.  The
// launch also moves the rings on (the pass in front has read them).
// --------------------------------------------------------------------------
template <int NQ, int PF>
__global__ __launch_bounds__(SS_SCAN_WAVES * TK_WAVE) void ss_scan_kernel(SsArgs a, const float* __restrict__ rec, int ld_rec, int np,
                                                                              const float2* __restrict__ step) {
  const int h = blockIdx.x, r = blockIdx.y;
  const int first = a.q_start[r], last = a.q_start[r + 1];
  if (first >= last) return;
  float* slot = a.state + (size_t)a.slots[r] * a.state_stride;
  ss_move_ring(a, slot, first, last, (blockIdx.z * gridDim.x + h) * blockDim.x + threadIdx.x, gridDim.x * gridDim.z * blockDim.x);
  const int lane = threadIdx.x % SS_LANES, grp = threadIdx.x / SS_LANES;
  const int col = blockIdx.z * (blockDim.x / SS_LANES) + grp;
  if ((col / SS_COLS) * SS_COLS >= a.dv) return;  // a wavefront none of whose columns exists
  const bool live = col < a.dv;
  const int N = a.N, inner = a.H * a.dv, g = h / (a.H / a.G);
  float* s_col = slot + ((size_t)h * a.dv + (live ? col : 0)) * N;
  const bool vec = (N % 4 == 0) && (a.state_stride % 4 == 0);
  float s[NQ][4];
#pragma unroll
  for (int n = 0; n < NQ; ++n) {
    const int i = 4 * (lane + SS_LANES * n);
    if (vec && live && i < N) {
      const float4 v = *(const float4*)(s_col + i);
      s[n][0] = v.x; s[n][1] = v.y; s[n][2] = v.z; s[n][3] = v.w;
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e) s[n][e] = (live && i + e < N) ? s_col[i + e] : 0.f;
    }
  }
  const int b_at = ss_rec_b(inner) + g * np + 4 * lane, c_at = b_at + a.G * np;
  const int x_at = h * a.dv + (live ? col : 0);
  const float dd = a.d_skip[h];

  float4 bv[2][PF][NQ], cv[2][PF][NQ];
  float xv[2][PF];
  float2 ev[2][PF];
  // rows of tokens t0 .. t0 + PF - 1 (those beyond the request's end repeat its last token and are not used)
#define SS_LOAD(Q, T0)                                                               \
  _Pragma("unroll") for (int j = 0; j < PF; ++j) {                                   \
    const size_t tok = min((T0) + j, last - 1);                                      \
    const float* row = rec + tok * ld_rec;                                           \
    _Pragma("unroll") for (int n = 0; n < NQ; ++n) {                                 \
      bv[Q][j][n] = *(const float4*)(row + b_at + 4 * SS_LANES * n);                 \
      cv[Q][j][n] = *(const float4*)(row + c_at + 4 * SS_LANES * n);                 \
    }                                                                                \
    xv[Q][j] = row[x_at];                                                            \
    ev[Q][j] = step[tok * a.H + h];                                                  \
  }
#define SS_STEP(Q, T0)                                                               \
  _Pragma("unroll") for (int j = 0; j < PF; ++j) {                                   \
    if ((T0) + j < last) {                                                           \
      const float xx = xv[Q][j], da = ev[Q][j].x, vv = ev[Q][j].y * xx;              \
      float acc0 = 0.f, acc1 = 0.f;                                                  \
      _Pragma("unroll") for (int n = 0; n < NQ; ++n) {                               \
        const float bb[4] = {bv[Q][j][n].x, bv[Q][j][n].y, bv[Q][j][n].z, bv[Q][j][n].w}; \
        const float cc[4] = {cv[Q][j][n].x, cv[Q][j][n].y, cv[Q][j][n].z, cv[Q][j][n].w}; \
        _Pragma("unroll") for (int e = 0; e < 4; ++e) s[n][e] = fmaf(da, s[n][e], bb[e] * vv); \
        acc0 = fmaf(cc[0], s[n][0], acc0); acc1 = fmaf(cc[1], s[n][1], acc1);        \
        acc0 = fmaf(cc[2], s[n][2], acc0); acc1 = fmaf(cc[3], s[n][3], acc1);        \
      }                                                                              \
      const float sum = row_sum16(acc0 + acc1);                                      \
      if (live && lane == 0) a.y[(size_t)((T0) + j) * inner + (size_t)h * a.dv + col] = fmaf(dd, xx, sum); \
    }                                                                                \
  }
  SS_LOAD(0, first);
#pragma unroll 1
  for (int t0 = first; t0 < last; t0 += 2 * PF) {
    SS_LOAD(1, t0 + PF);
    SS_STEP(0, t0);
    SS_LOAD(0, t0 + 2 * PF);
    SS_STEP(1, t0 + PF);
  }
#undef SS_LOAD
#undef SS_STEP
  if (!live) return;
#pragma unroll
  for (int n = 0; n < NQ; ++n) {
    const int i = 4 * (lane + SS_LANES * n);
    if (vec && i < N) {
      *(float4*)(s_col + i) = make_float4(s[n][0], s[n][1], s[n][2], s[n][3]);
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (i + e < N) s_col[i + e] = s[n][e];
    }
  }
}

// --------------------------------------------------------------------------
// Chunks of SS_CHUNK tokens of a request's portion.  With l_t the sum of the decays' logarithms from the chunk's first
// token to token t, and S the state in front of the chunk,
//     y_t = exp(l_t) C_t S + sum_{s <= t} (C_t . B_s) exp(l_t - l_s) dt_s x_s + D x_t
//     S  <- exp(l_last) S + sum_s exp(l_last - l_s) dt_s B_s x_s^T
// All exponents are at most 0.  C . B is a product of bfloat16 numbers (exact, 32-bit sums, v_mfma_f32_16x16x32_bf16);
// every other product has a 32-bit operand and runs on the 32-bit matrix cores (v_mfma_f32_16x16x4_f32).
//
// A workgroup owns 16 value columns of one (head, request) and walks its chunks; its four wavefronts take the chunk's
// four tiles of 16 tokens each for y (wavefront w sees token tiles 0 .. w), and the rows of S 32 at a time for the
// update (wavefront w the 32s w, w + 4, ..: row 8 c + 2 i + T of a 32 is row 4 c + i of product tile T, so that a lane
// reads two neighbouring numbers of B and ends up with eight neighbouring rows of S).  S stays in registers; every
// chunk also hands it to the other wavefronts through LDS, [row / 8][column][8].  A chunk's rows of B, C and x are
// asked for while the chunk before is computed, and put into LDS (rows padded by 16 bytes) between two barriers.
// NM: row pieces of 32 (np / 32), NP: those of one wavefront.
// --------------------------------------------------------------------------
#define SS_CHUNK 64
#define SS_LOG2E 1.44269504088896341f

template <int NM, int NP>
__global__ __launch_bounds__(4 * TK_WAVE) void ss_chunk_kernel(SsArgs a, const bf16_t* __restrict__ rec, int ld_rec,
                                                               const float2* __restrict__ step) {
  constexpr int NROWS = NM * 32;
  constexpr int LD = 2 * NROWS + 8;     // a row of bc: [B | C], and the padding
  constexpr int LDX = 20;               // a row of xs
  constexpr int PIECES = 2 * NROWS / 8;  // 16-byte pieces of a row
  constexpr int PER = SS_CHUNK * PIECES / 256;
  __shared__ __align__(16) bf16_t bc[SS_CHUNK * LD];
  __shared__ bf16_t xs[SS_CHUNK * LDX];
  __shared__ __align__(16) float s_lds[NROWS * 16];
  __shared__ __align__(16) float l_lds[SS_CHUNK], dt_lds[SS_CHUNK];  // the sums of the logarithms, to base 2
  // neighbouring workgroups go to different dies: the heads of a group then share one die's cache
  const int h = a.H % 8 == 0 ? (blockIdx.x % 8) * (a.H / 8) + blockIdx.x / 8 : blockIdx.x;
  const int r = blockIdx.y;
  const int first = a.q_start[r], last = a.q_start[r + 1];
  if (first >= last) return;
  float* slot = a.state + (size_t)a.slots[r] * a.state_stride;
  ss_move_ring(a, slot, first, last, (blockIdx.z * gridDim.x + blockIdx.x) * blockDim.x + threadIdx.x, gridDim.x * gridDim.z * blockDim.x);
  const int lane = threadIdx.x & (TK_WAVE - 1), wave = __builtin_amdgcn_readfirstlane(threadIdx.x / TK_WAVE);
  const int col = lane & 15, c = lane >> 4;
  const int j0 = blockIdx.z * 16, j = j0 + col;
  const bool live = j < a.dv;
  const int N = a.N, inner = a.H * a.dv, g = h / (a.H / a.G);
  const int b_at = ss_rec_b(inner) + g * NROWS;
  const float dd = a.d_skip[h];
  float* s_col = slot + ((size_t)h * a.dv + (live ? j : 0)) * N;  // this lane's column of the state in memory

  // the state: row 32 (wave + 4 p) + 8 c + 2 i + T of column j is sv[p][T][i]
  v4f sv[NP][2];
#pragma unroll
  for (int p = 0; p < NP; ++p)
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int T = 0; T < 2; ++T) {
        const int n = 32 * (wave + 4 * p) + 8 * c + 2 * i + T;
        sv[p][T][i] = live && n < N ? s_col[n] : 0.f;
      }
  // what a thread brings of the next chunk: pieces of its rows of B and C, four numbers of x, and (first wavefront) a
  // token's step.  Tokens beyond the request's end repeat the last one's row and have no step and no decay.
  u32x4 pre[PER];
  bf16_t prex[4];
  float2 mine;
  auto ask = [&](int t0) {
#pragma unroll
    for (int k = 0; k < PER; ++k) {
      const int i = threadIdx.x + 256 * k, row = i / PIECES, piece = i % PIECES;
      const bf16_t* src = rec + (size_t)min(t0 + row, last - 1) * ld_rec + b_at;
      pre[k] = *(const u32x4*)(src + (piece < NROWS / 8 ? piece * 8 : a.G * NROWS + piece * 8 - NROWS));
    }
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      const int i = threadIdx.x + 256 * k, row = i / 16, x = j0 + i % 16;
      prex[k] = rec[(size_t)min(t0 + row, last - 1) * ld_rec + h * a.dv + min(x, a.dv - 1)];
    }
    if (wave == 0) mine = t0 + lane < last ? step[(size_t)(t0 + lane) * a.H + h] : make_float2(0.f, 0.f);
  };
  auto put = [&]() {
#pragma unroll
    for (int k = 0; k < PER; ++k) {
      const int i = threadIdx.x + 256 * k, row = i / PIECES, piece = i % PIECES;
      *(u32x4*)(bc + row * LD + piece * 8) = pre[k];
    }
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      const int i = threadIdx.x + 256 * k;
      xs[(i / 16) * LDX + i % 16] = prex[k];
    }
#pragma unroll
    for (int p = 0; p < NP; ++p) {
      const int piece = 4 * (wave + 4 * p) + c;
      if (piece * 8 < NROWS) {
        float4* d = (float4*)(s_lds + (piece * 16 + col) * 8);
        d[0] = make_float4(sv[p][0][0], sv[p][1][0], sv[p][0][1], sv[p][1][1]);
        d[1] = make_float4(sv[p][0][2], sv[p][1][2], sv[p][0][3], sv[p][1][3]);
      }
    }
    if (wave == 0) {
      float l = mine.x;
#pragma unroll
      for (int o = 1; o < SS_CHUNK; o <<= 1) {
        const float up = __shfl_up(l, o, TK_WAVE);
        if (lane >= o) l += up;
      }
      l_lds[lane] = l * SS_LOG2E;
      dt_lds[lane] = mine.y;
    }
  };
  ask(first);
  put();
  __syncthreads();
#pragma unroll 1
  for (int t0 = first; t0 < last; t0 += SS_CHUNK) {
    const bool more = t0 + SS_CHUNK < last;
    if (more) ask(t0 + SS_CHUNK);
    bf16x8_t cv[NM];  // C of token 16 wave + col
    float xv[4][4];   // x of tokens 16 T + 4 c + i
#pragma unroll
    for (int m = 0; m < NM; ++m) cv[m] = *(const bf16x8_t*)(bc + (16 * wave + col) * LD + NROWS + 32 * m + 8 * c);
#pragma unroll
    for (int T = 0; T < 4; ++T)
#pragma unroll
      for (int i = 0; i < 4; ++i) xv[T][i] = to_f32<bf16_t>(xs[(16 * T + 4 * c + i) * LDX + col]);
    // y: what the state in front of the chunk gives its tokens
    v4f y = (v4f){0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int m = 0; m < NM; ++m) {
      const float4* sp = (const float4*)(s_lds + ((4 * m + c) * 16 + col) * 8);
      const float4 s0 = sp[0], s1 = sp[1];
      const float sr[8] = {s0.x, s0.y, s0.z, s0.w, s1.x, s1.y, s1.z, s1.w};
#pragma unroll
      for (int e = 0; e < 8; ++e) y = __builtin_amdgcn_mfma_f32_16x16x4f32((float)cv[m][e], sr[e], y, 0, 0, 0);
    }
    {
      const float4 lt = *(const float4*)(l_lds + 16 * wave + 4 * c);
      y[0] *= __builtin_amdgcn_exp2f(lt.x); y[1] *= __builtin_amdgcn_exp2f(lt.y); y[2] *= __builtin_amdgcn_exp2f(lt.z); y[3] *= __builtin_amdgcn_exp2f(lt.w);
    }
    // y: what the chunk's own tokens give each other; the lane of token t holds tokens s = 16 T + 4 c + i
    const float l_t = l_lds[16 * wave + col], l_end = l_lds[SS_CHUNK - 1];
    float ws[4][4];  // the weights of the state's update
#pragma unroll
    for (int T = 0; T < 4; ++T) {
      const float4 ls = *(const float4*)(l_lds + 16 * T + 4 * c), ds = *(const float4*)(dt_lds + 16 * T + 4 * c);
      const float lv[4] = {ls.x, ls.y, ls.z, ls.w}, dv4[4] = {ds.x, ds.y, ds.z, ds.w};
#pragma unroll
      for (int i = 0; i < 4; ++i) ws[T][i] = __builtin_amdgcn_exp2f(l_end - lv[i]) * dv4[i] * xv[T][i];
      if (T > wave) continue;  // (the same for all lanes)
      v4f gm = (v4f){0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int m = 0; m < NM; ++m)
        gm = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*(const bf16x8_t*)(bc + (16 * T + col) * LD + 32 * m + 8 * c), cv[m], gm, 0, 0, 0);
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const bool seen = T < wave || 4 * c + i <= col;
        const float w = gm[i] * (__builtin_amdgcn_exp2f(seen ? l_t - lv[i] : -INFINITY) * dv4[i]);
        y = __builtin_amdgcn_mfma_f32_16x16x4f32(w, xv[T][i], y, 0, 0, 0);
      }
      if (T == wave) {
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int t = t0 + 16 * T + 4 * c + i;
          if (live && t < last) a.y[(size_t)t * inner + (size_t)h * a.dv + j] = fmaf(dd, xv[T][i], y[i]);
        }
      }
    }
    // the state behind the chunk
    const float keep = __builtin_amdgcn_exp2f(l_end);
#pragma unroll
    for (int p = 0; p < NP; ++p) {
      const int n = 32 * (wave + 4 * p) + 2 * col;
      if (32 * (wave + 4 * p) >= NROWS) continue;  // (the same for all lanes)
      sv[p][0] = sv[p][0] * keep;
      sv[p][1] = sv[p][1] * keep;
#pragma unroll
      for (int T = 0; T < 4; ++T)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const uint32_t two = *(const uint32_t*)(bc + (16 * T + 4 * c + i) * LD + n);
          sv[p][0] = __builtin_amdgcn_mfma_f32_16x16x4f32(__uint_as_float(two << 16), ws[T][i], sv[p][0], 0, 0, 0);
          sv[p][1] = __builtin_amdgcn_mfma_f32_16x16x4f32(__uint_as_float(two & 0xffff0000u), ws[T][i], sv[p][1], 0, 0, 0);
        }
    }
    __syncthreads();
    if (more) {
      put();
      __syncthreads();
    }
  }
  if (!live) return;
#pragma unroll
  for (int p = 0; p < NP; ++p)
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int T = 0; T < 2; ++T) {
        const int n = 32 * (wave + 4 * p) + 8 * c + 2 * i + T;
        if (n < N) s_col[n] = sv[p][T][i];
      }
}

// --------------------------------------------------------------------------
// A step in which every request brings one token: one kernel.  A workgroup (head, request, block of columns) asks for
// its part of the state, computes the convolution of its columns of x and of its group's B and C into LDS, and takes
// the recurrence one token on, with the functions and the order of the kernels above (the same bits).  The ring's new
// entries are written by the workgroups of a group's first head (B, C) and by a column's own (x).
// --------------------------------------------------------------------------
template <int NQ>
__global__ __launch_bounds__(SS_WAVES * TK_WAVE) void ss_single_kernel(SsArgs a) {
  __shared__ float bs[NQ * 64], cs[NQ * 64], xs[SS_WAVES * SS_COLS], es[2];
  const int h = blockIdx.x, r = blockIdx.y;
  const int t = a.q_start[r];
  if (a.q_start[r + 1] <= t) return;
  const int lane = threadIdx.x % SS_LANES, grp = threadIdx.x / SS_LANES;
  const int cols = blockDim.x / SS_LANES, col0 = blockIdx.z * cols, col = col0 + grp;
  const bool live = col < a.dv;
  const int N = a.N, inner = a.H * a.dv, heads_a_group = a.H / a.G, g = h / heads_a_group;
  float* slot = a.state + (size_t)a.slots[r] * a.state_stride;
  float* s_col = slot + ((size_t)h * a.dv + (live ? col : 0)) * N;
  const bool vec = (N % 4 == 0) && (a.state_stride % 4 == 0);
  float s[NQ][4];
#pragma unroll
  for (int n = 0; n < NQ; ++n) {
    const int i = 4 * (lane + SS_LANES * n);
    if (vec && live && i < N) {
      const float4 v = *(const float4*)(s_col + i);
      s[n][0] = v.x; s[n][1] = v.y; s[n][2] = v.z; s[n][3] = v.w;
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e) s[n][e] = (live && i + e < N) ? s_col[i + e] : 0.f;
    }
  }
  const int pos = a.positions[t];
  float* ring = slot + a.ring_off;
  const int n_x = min(cols, a.dv - col0);
  for (int i = threadIdx.x; i < 2 * NQ * 64 + n_x; i += blockDim.x) {
    int c;
    bool writer;
    if (i < 2 * NQ * 64) {
      const int part = i / (NQ * 64), k = i % (NQ * 64);
      if (k >= N) {
        (part ? cs : bs)[k] = 0.f;
        continue;
      }
      c = inner + (part * a.G + g) * N + k;
      writer = h % heads_a_group == 0 && blockIdx.z == 0;
      (part ? cs : bs)[k] = ss_channel(a, t, 0, pos, ring, c);
    } else {
      const int k = i - 2 * NQ * 64;
      c = h * a.dv + col0 + k;
      writer = true;
      xs[k] = ss_channel(a, t, 0, pos, ring, c);
    }
    if (writer && a.taps > 1) ring[(size_t)(pos % a.taps) * a.channels + c] = a.proj[(size_t)t * a.ld + a.x_off + c];
  }
  if (threadIdx.x == 0) {
    const float dt = ss_softplus(a.proj[(size_t)t * a.ld + a.dt_off + h] + a.dt_bias[h]);
    es[0] = ss_decay(a.a_log[h], dt);
    es[1] = dt;
  }
  __syncthreads();
  const float xx = live ? xs[grp] : 0.f, da = es[0], vv = es[1] * xx;
  float acc0 = 0.f, acc1 = 0.f;
#pragma unroll
  for (int n = 0; n < NQ; ++n) {
    const int i = 4 * (lane + SS_LANES * n);
    const float4 b4 = *(const float4*)(bs + i), c4 = *(const float4*)(cs + i);
    const float bb[4] = {b4.x, b4.y, b4.z, b4.w}, cc[4] = {c4.x, c4.y, c4.z, c4.w};
#pragma unroll
    for (int e = 0; e < 4; ++e) s[n][e] = fmaf(da, s[n][e], bb[e] * vv);
    acc0 = fmaf(cc[0], s[n][0], acc0); acc1 = fmaf(cc[1], s[n][1], acc1);
    acc0 = fmaf(cc[2], s[n][2], acc0); acc1 = fmaf(cc[3], s[n][3], acc1);
  }
  const float sum = row_sum16(acc0 + acc1);
  if (!live) return;
  if (lane == 0) a.y[(size_t)t * inner + (size_t)h * a.dv + col] = fmaf(a.d_skip[h], xx, sum);
#pragma unroll
  for (int n = 0; n < NQ; ++n) {
    const int i = 4 * (lane + SS_LANES * n);
    if (vec && i < N) {
      *(float4*)(s_col + i) = make_float4(s[n][0], s[n][1], s[n][2], s[n][3]);
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (i + e < N) s_col[i + e] = s[n][e];
    }
  }
}

enum { SS_SINGLE = 0, SS_SCAN = 1, SS_CHUNKS = 2 };
#define SS_CHUNKS_FROM 16  // tokens of a step's longest portion from which on it goes in chunks
static int ss_form(int dt, int N, int longest) {
  if (longest <= 1) return SS_SINGLE;
  return dt == TK_BF16 && longest >= SS_CHUNKS_FROM && N <= 256 ? SS_CHUNKS : SS_SCAN;
}
static int ss_padded(int form, int N) {
  if (form == SS_SCAN) return 64 * ss_pieces(N);
  const int nm = (N + 31) / 32;
  return 32 * (nm <= 4 ? nm : (nm <= 6 ? 6 : 8));
}
// Bytes of working memory that a step takes for every token.
TK_API int tk_state_space_token_bytes(int dt, int H, int G, int N, int dv, int longest) {
  const int form = ss_form(dt, N, longest);
  if (form == SS_SINGLE) return 0;
  return ss_rec_width(H * dv, G, ss_padded(form, N)) * (form == SS_SCAN ? 4 : 2) + 8 * H;
}

TK_API int tk_state_space(int dt, const float* proj, int ld, int x_off, int dt_off, const float* conv_w, const float* conv_b, int taps,
                          const float* a_log, const float* dt_bias, const float* d_skip, float* state, size_t state_stride,
                          size_t ring_off, const int* q_start, const int* token_req, const int* slots, const int* positions,
                          void* work, float* y, int n_tokens, int n_requests, int H, int G, int N, int dv, int longest,
                          hipStream_t stream) {
  TK_REQUIRE(n_tokens >= 0 && n_requests >= 0 && H > 0 && G > 0 && H % G == 0 && N > 0 && N <= 512 && dv > 0 && taps >= 1,
             "state_space: bad sizes tokens=%d requests=%d heads=%d groups=%d state=%d dv=%d taps=%d (state up to 512)", n_tokens,
             n_requests, H, G, N, dv, taps);
  const int channels = H * dv + 2 * G * N, inner = H * dv;
  TK_REQUIRE(x_off >= 0 && x_off + channels <= ld && dt_off >= 0 && dt_off + H <= ld, "state_space: a part lies outside the rows");
  TK_REQUIRE(longest >= 1, "state_space: the longest portion of a step with tokens is at least one token");
  const int form = ss_form(dt, N, longest);
  TK_REQUIRE(proj && conv_w && conv_b && a_log && dt_bias && d_skip && state && q_start && token_req && slots && positions && y &&
                 (work || form == SS_SINGLE),
             "state_space: a pointer is missing");
  TK_REQUIRE(ring_off >= (size_t)H * dv * N && state_stride >= ring_off + (taps > 1 ? (size_t)taps * channels : 0),
             "state_space: the state's rows are too short");
  TK_REQUIRE((((uintptr_t)work | (uintptr_t)state) & 15) == 0, "state_space: working memory and state must start at multiples of 16 bytes");
  TK_REQUIRE(n_requests < 65536 && n_tokens < 65536 && dv <= 65535, "state_space: the step is too large");
  if (n_requests == 0 || n_tokens == 0) return 0;
  const SsArgs a{proj, ld, x_off, dt_off, conv_w, conv_b, taps, channels, a_log, dt_bias, d_skip, state, state_stride, ring_off,
                 q_start, token_req, slots, positions, y, H, G, N, dv, dt == TK_BF16 ? 1 : 0};
  const int waves_all = (dv + SS_COLS - 1) / SS_COLS;  // wavefronts that the columns of a head take, token by token
  const int nq = ss_pieces(N);
  if (form == SS_SINGLE) {
    const int waves = min(SS_WAVES, waves_all);
    const dim3 grid(H, n_requests, (waves_all + waves - 1) / waves), block(waves * TK_WAVE);
#define SS_ONE(NQ) hipLaunchKernelGGL((ss_single_kernel<NQ>), grid, block, 0, stream, a)
    if (nq <= 1) SS_ONE(1);
    else if (nq <= 2) SS_ONE(2);
    else if (nq <= 3) SS_ONE(3);
    else if (nq <= 4) SS_ONE(4);
    else if (nq <= 6) SS_ONE(6);
    else SS_ONE(8);
#undef SS_ONE
    TK_CHECK_LAUNCH("state_space");
    return 0;
  }
  const int np = ss_padded(form, N), ld_rec = ss_rec_width(inner, G, np);
  float2* step = (float2*)((char*)work + (size_t)n_tokens * ld_rec * (form == SS_SCAN ? 4 : 2));  // (rows are multiples of 16 bytes)
  const bool vec = inner % 4 == 0 && N % 4 == 0 && ld % 4 == 0 && x_off % 4 == 0 && state_stride % 4 == 0 && ring_off % 4 == 0 &&
                   (((uintptr_t)proj | (uintptr_t)conv_w | (uintptr_t)conv_b) & 15) == 0;
  const int items = vec ? ld_rec / 4 + H : ld_rec + H;
  const dim3 pgrid((items + 255) / 256, n_tokens);
#define SS_PREPARE(T, V) \
  hipLaunchKernelGGL((ss_prepare_kernel<T, V>), pgrid, dim3(256), 0, stream, a, (T*)work, ld_rec, np, step, form == SS_CHUNKS)
  if (form == SS_SCAN) {
    if (vec) SS_PREPARE(float, 4); else SS_PREPARE(float, 1);
  } else {
    if (vec) SS_PREPARE(bf16_t, 4); else SS_PREPARE(bf16_t, 1);
  }
#undef SS_PREPARE
  if (form == SS_CHUNKS) {
    const dim3 grid(H, n_requests, (dv + 15) / 16);
#define SS_CASE(NM, NP) hipLaunchKernelGGL((ss_chunk_kernel<NM, NP>), grid, dim3(4 * TK_WAVE), 0, stream, a, (const bf16_t*)work, ld_rec, step)
    switch (np / 32) {
      case 1: SS_CASE(1, 1); break;
      case 2: SS_CASE(2, 1); break;
      case 3: SS_CASE(3, 1); break;
      case 4: SS_CASE(4, 1); break;
      case 6: SS_CASE(6, 2); break;
      default: SS_CASE(8, 2); break;
    }
#undef SS_CASE
    TK_CHECK_LAUNCH("state_space");
    return 0;
  }
  // A long walk is a chain of arithmetic in every wavefront: one wavefront a workgroup then spreads a prompt over all
  // compute units.  Steps of few tokens a request launch many short wavefronts, in workgroups of several.
  const int waves = longest > 16 ? 1 : min(SS_SCAN_WAVES, waves_all);
  const dim3 grid(H, n_requests, (waves_all + waves - 1) / waves), block(waves * TK_WAVE);
#define SS_CASE(NQ, PF) hipLaunchKernelGGL((ss_scan_kernel<NQ, PF>), grid, block, 0, stream, a, (const float*)work, ld_rec, np, step)
  if (nq <= 1) SS_CASE(1, 4);
  else if (nq <= 2) SS_CASE(2, 4);
  else if (nq <= 3) SS_CASE(3, 2);
  else if (nq <= 4) SS_CASE(4, 2);
  else if (nq <= 6) SS_CASE(6, 1);
  else SS_CASE(8, 1);
#undef SS_CASE
  TK_CHECK_LAUNCH("state_space");
  return 0;
}

// --------------------------------------------------------------------------
// v = y * silu(z); every one of `groups` equal parts of a row of v divided by its own root mean square, times the
// row's weight w [groups * size]; rounded once to T.  The gate comes before the norm.  A workgroup a (token, part);
// parts of up to 4 * 256 * GN_QUADS numbers in whole 16-byte pieces stay in registers between the two passes.
// --------------------------------------------------------------------------
#define GN_QUADS 8
template <typename T>
__global__ __launch_bounds__(256) void gate_group_norm_kernel(const float* __restrict__ y, const float* __restrict__ z, int ld_z,
                                                              const float* __restrict__ w, float eps, T* __restrict__ out, int groups,
                                                              int size, int vec) {
  __shared__ float red[16];
  const size_t t = blockIdx.x / groups;
  const int g = blockIdx.x % groups;
  const float* yr = y + (t * groups + g) * size;
  const float* zr = z + t * ld_z + (size_t)g * size;
  const float* wr = w + (size_t)g * size;
  T* dst = out + (t * groups + g) * size;
  float ss = 0.f;
  if (vec) {
    float4 v[GN_QUADS];
#pragma unroll
    for (int q = 0; q < GN_QUADS; ++q) {
      const int i = threadIdx.x + q * blockDim.x;
      if (i < size / 4) {
        const float4 a = ((const float4*)yr)[i], b = ((const float4*)zr)[i];
        v[q] = make_float4(a.x * ss_silu(b.x), a.y * ss_silu(b.y), a.z * ss_silu(b.z), a.w * ss_silu(b.w));
        ss = fmaf(v[q].x, v[q].x, ss); ss = fmaf(v[q].y, v[q].y, ss); ss = fmaf(v[q].z, v[q].z, ss); ss = fmaf(v[q].w, v[q].w, ss);
      }
    }
    const float rstd = 1.0f / sqrtf(block_sum(ss, red) / (float)size + eps);
#pragma unroll
    for (int q = 0; q < GN_QUADS; ++q) {
      const int i = threadIdx.x + q * blockDim.x;
      if (i < size / 4) {
        const float4 k = ((const float4*)wr)[i];
        struct alignas(sizeof(T) * 4) Quad { T v[4]; } o;
        o.v[0] = from_f32<T>(v[q].x * rstd * k.x);
        o.v[1] = from_f32<T>(v[q].y * rstd * k.y);
        o.v[2] = from_f32<T>(v[q].z * rstd * k.z);
        o.v[3] = from_f32<T>(v[q].w * rstd * k.w);
        ((Quad*)dst)[i] = o;
      }
    }
    return;
  }
  for (int i = threadIdx.x; i < size; i += blockDim.x) {
    const float v = yr[i] * ss_silu(zr[i]);
    ss = fmaf(v, v, ss);
  }
  const float rstd = 1.0f / sqrtf(block_sum(ss, red) / (float)size + eps);
  for (int i = threadIdx.x; i < size; i += blockDim.x) dst[i] = from_f32<T>(yr[i] * ss_silu(zr[i]) * rstd * wr[i]);
}

TK_API int tk_gate_group_norm(int dt, const float* y, const float* z, int ld_z, const float* w, float eps, void* out, int n_tokens,
                              int groups, int size, hipStream_t stream) {
  TK_REQUIRE(n_tokens >= 0 && groups > 0 && size > 0 && y && z && w && out && ld_z >= groups * size,
             "gate_group_norm: bad sizes %d %d %d, a pointer is missing or the gate's rows are too short", n_tokens, groups, size);
  TK_REQUIRE((long)n_tokens * groups < (1l << 31), "gate_group_norm: too many rows");
  if (n_tokens == 0) return 0;
  const int vec = size % 4 == 0 && size <= 4 * 256 * GN_QUADS && ld_z % 4 == 0 &&
                  (((uintptr_t)y | (uintptr_t)z | (uintptr_t)w | (uintptr_t)out) & 15) == 0;
  const int work = vec ? size / 4 : size;
  const int threads = work <= 64 ? 64 : (work <= 128 ? 128 : 256);
  const dim3 grid(n_tokens * groups);
  if (dt == TK_F32)
    hipLaunchKernelGGL(gate_group_norm_kernel<float>, grid, dim3(threads), 0, stream, y, z, ld_z, w, eps, (float*)out, groups, size, vec);
  else
    hipLaunchKernelGGL(gate_group_norm_kernel<bf16_t>, grid, dim3(threads), 0, stream, y, z, ld_z, w, eps, (bf16_t*)out, groups, size, vec);
  TK_CHECK_LAUNCH("gate_group_norm");
  return 0;
}
