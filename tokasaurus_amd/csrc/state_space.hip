// A selective state-space mixer (Mamba-2's form) as a recurrence over the tokens of each request, and the gated norm
// behind it.  Per head, with a matrix S [N][dv] kept per request in 32-bit and B, C shared by the heads of a group:
//     u = silu(conv(.)) for x | B | C       a causal convolution over time on every channel, with a bias
//     dt = softplus(. + dt_bias[h])         a = exp(-exp(A_log[h]) dt)
//     S <- a S + dt B x^T                   y = S^T C + D[h] x
// All of it is read from the 32-bit sums `proj` of one stacked product (x | B | C are `channels` neighbouring columns,
// dt another H) and is 32-bit arithmetic.
//
// What a slot keeps: [H][dv][N] the matrices (a value column's N numbers lie together), and from `ring_off` on the
// convolution's last inputs as a ring [taps][channels]: the input of position p lies in entry p % taps.  A token needs
// the entries of the taps - 1 positions before it and never the one that it writes, so workgroups that read the same
// channels need no order among themselves.  Positions in front of a request's start count as zeros.
//
// The columns of S do not meet: a column is owned by SS_LANES neighbouring lanes that cut N between them and add up
// through the wavefront's own data paths, always in the same order, so a token's result does not depend on how its
// request's tokens were cut into steps or on what shares the batch.
#include "common.h"

#define SS_LANES 16
#define SS_COLS 4    // value columns a wavefront owns
#define SS_WAVES 16  // most wavefronts of a workgroup

__device__ __forceinline__ float ss_silu(float x) { return x / (1.0f + expf(-x)); }
__device__ __forceinline__ float ss_softplus(float x) { return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))); }
__device__ __forceinline__ float ss_decay(float a_log, float dt) { return expf(-__fmul_rn(expf(a_log), dt)); }

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
  return ss_silu(acc);
}

// 16-byte pieces of a column that a lane holds: one of the kernels' instances (1, 2, 3, 4, 6, 8)
static int ss_pieces(int n) {
  const int nq = (n + 63) / 64;
  return nq <= 4 ? nq : (nq <= 6 ? 6 : 8);
}
// where the parts of a row of `rec` begin: [x: inner | B: G x np | C: G x np | (a, dt): H x 2], np = 64 times the pieces
// a lane holds, zeros in the padding (a padded row of S meets a zero of C)
__host__ __device__ __forceinline__ int ss_rec_b(int inner) { return (inner + 3) / 4 * 4; }
__host__ __device__ __forceinline__ int ss_rec_width(int inner, int G, int np, int H) { return ss_rec_b(inner) + 2 * G * np + (2 * H + 3) / 4 * 4; }

// --------------------------------------------------------------------------
// Before the recurrence of a step with portions, once a token: convolution, activations, step sizes and decays.
// --------------------------------------------------------------------------
__global__ __launch_bounds__(256) void ss_prepare_kernel(SsArgs a, float* __restrict__ rec, int ld_rec, int np) {
  const int t = blockIdx.y;
  const int x = blockIdx.x * blockDim.x + threadIdx.x;
  if (x >= ld_rec) return;
  const int inner = a.H * a.dv, b0 = ss_rec_b(inner), e0 = b0 + 2 * a.G * np;
  const int r = a.token_req[t];
  const int local = t - a.q_start[r];
  const float* ring = a.state + (size_t)a.slots[r] * a.state_stride + a.ring_off;
  float v = 0.f;
  if (x < b0) {
    if (x < inner) v = ss_channel(a, t, local, a.positions[t], ring, x);
  } else if (x < e0) {
    const int g = (x - b0) / np, i = (x - b0) % np;  // g counts the groups of B, then those of C
    if (i < a.N) v = ss_channel(a, t, local, a.positions[t], ring, inner + g * a.N + i);
  } else if (x < e0 + 2 * a.H) {
    const int h = (x - e0) / 2;
    const float dt = ss_softplus(a.proj[(size_t)t * a.ld + a.dt_off + h] + a.dt_bias[h]);
    v = (x - e0) % 2 ? dt : ss_decay(a.a_log[h], dt);
  }
  rec[(size_t)t * ld_rec + x] = v;
}

// --------------------------------------------------------------------------
// The recurrence of a step with portions.  A wavefront owns SS_COLS value columns of one (head, request); lane l of a
// column's SS_LANES holds rows 4 * (l + SS_LANES * n) + e, n < NQ, e < 4.  No LDS and no barrier: the wavefronts of a
// group's heads read the same rows of `rec` through the caches, two groups of PF tokens ahead of the arithmetic.  The
// launch also moves the rings on (the pass in front has read them).
// --------------------------------------------------------------------------
template <int NQ, int PF>
__global__ __launch_bounds__(SS_WAVES * TK_WAVE) void ss_scan_kernel(SsArgs a, const float* __restrict__ rec, int ld_rec, int np) {
  const int h = blockIdx.x, r = blockIdx.y;
  const int first = a.q_start[r], last = a.q_start[r + 1];
  if (first >= last) return;
  float* slot = a.state + (size_t)a.slots[r] * a.state_stride;
  if (a.taps > 1) {
    // the last `taps` inputs of the step's tokens (fewer when it brings fewer; the rest of the ring stays)
    const int threads = gridDim.x * gridDim.z * blockDim.x;
    for (int c = (blockIdx.z * gridDim.x + h) * blockDim.x + threadIdx.x; c < a.channels; c += threads)
      for (int t = max(first, last - a.taps); t < last; ++t)
        slot[a.ring_off + (size_t)(a.positions[t] % a.taps) * a.channels + c] = a.proj[(size_t)t * a.ld + a.x_off + c];
  }
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
  const int x_at = h * a.dv + (live ? col : 0), e_at = ss_rec_b(inner) + 2 * a.G * np + 2 * h;
  const float dd = a.d_skip[h];

  float4 bv[2][PF][NQ], cv[2][PF][NQ];
  float xv[2][PF];
  float2 ev[2][PF];
  // rows of tokens t0 .. t0 + PF - 1 (those beyond the request's end repeat its last token and are not used)
#define SS_LOAD(Q, T0)                                                               \
  _Pragma("unroll") for (int j = 0; j < PF; ++j) {                                   \
    const float* row = rec + (size_t)min((T0) + j, last - 1) * ld_rec;               \
    _Pragma("unroll") for (int n = 0; n < NQ; ++n) {                                 \
      bv[Q][j][n] = *(const float4*)(row + b_at + 4 * SS_LANES * n);                 \
      cv[Q][j][n] = *(const float4*)(row + c_at + 4 * SS_LANES * n);                 \
    }                                                                                \
    xv[Q][j] = row[x_at];                                                            \
    ev[Q][j] = *(const float2*)(row + e_at);                                         \
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

// Floats of a row of `rec` for these sizes.
TK_API int tk_state_space_rec_width(int H, int G, int N, int dv) { return ss_rec_width(H * dv, G, 64 * ss_pieces(N), H); }

TK_API int tk_state_space(const float* proj, int ld, int x_off, int dt_off, const float* conv_w, const float* conv_b, int taps,
                          const float* a_log, const float* dt_bias, const float* d_skip, float* state, size_t state_stride,
                          size_t ring_off, const int* q_start, const int* token_req, const int* slots, const int* positions,
                          float* rec, float* y, int n_tokens, int n_requests, int H, int G, int N, int dv, int longest,
                          hipStream_t stream) {
  TK_REQUIRE(n_tokens >= 0 && n_requests >= 0 && H > 0 && G > 0 && H % G == 0 && N > 0 && N <= 512 && dv > 0 && taps >= 1,
             "state_space: bad sizes tokens=%d requests=%d heads=%d groups=%d state=%d dv=%d taps=%d (state up to 512)", n_tokens,
             n_requests, H, G, N, dv, taps);
  const int channels = H * dv + 2 * G * N;
  TK_REQUIRE(x_off >= 0 && x_off + channels <= ld && dt_off >= 0 && dt_off + H <= ld, "state_space: a part lies outside the rows");
  TK_REQUIRE(longest >= 1, "state_space: the longest portion of a step with tokens is at least one token");
  const bool single = longest == 1;
  TK_REQUIRE(proj && conv_w && conv_b && a_log && dt_bias && d_skip && state && q_start && token_req && slots && positions && y && (rec || single),
             "state_space: a pointer is missing");
  TK_REQUIRE(ring_off >= (size_t)H * dv * N && state_stride >= ring_off + (taps > 1 ? (size_t)taps * channels : 0),
             "state_space: the state's rows are too short");
  TK_REQUIRE((((uintptr_t)rec | (uintptr_t)state) & 15) == 0, "state_space: rec and state must start at multiples of 16 bytes");
  TK_REQUIRE(n_requests < 65536 && n_tokens < 65536 && dv <= 65535, "state_space: the step is too large");
  if (n_requests == 0 || n_tokens == 0) return 0;
  const SsArgs a{proj, ld, x_off, dt_off, conv_w, conv_b, taps, channels, a_log, dt_bias, d_skip, state, state_stride, ring_off,
                 q_start, token_req, slots, positions, y, H, G, N, dv};
  const int nq = ss_pieces(N), np = 64 * nq;
  const int waves_all = (dv + SS_COLS - 1) / SS_COLS;  // wavefronts that the columns of a head take
  if (single) {
    const int waves = min(SS_WAVES, waves_all);
    const dim3 grid(H, n_requests, (waves_all + waves - 1) / waves), block(waves * TK_WAVE);
#define SS_SINGLE(NQ) hipLaunchKernelGGL((ss_single_kernel<NQ>), grid, block, 0, stream, a)
    if (nq <= 1) SS_SINGLE(1);
    else if (nq <= 2) SS_SINGLE(2);
    else if (nq <= 3) SS_SINGLE(3);
    else if (nq <= 4) SS_SINGLE(4);
    else if (nq <= 6) SS_SINGLE(6);
    else SS_SINGLE(8);
#undef SS_SINGLE
    TK_CHECK_LAUNCH("state_space");
    return 0;
  }
  const int ld_rec = ss_rec_width(H * dv, G, np, H);
  hipLaunchKernelGGL(ss_prepare_kernel, dim3((ld_rec + 255) / 256, n_tokens), dim3(256), 0, stream, a, rec, ld_rec, np);
  // A long walk is a chain of arithmetic in every wavefront: one wavefront a workgroup then spreads a prompt over all
  // compute units.  Steps of few tokens a request launch many short wavefronts, in workgroups of several.
  const int waves = longest > 16 ? 1 : min(8, waves_all);
  const dim3 grid(H, n_requests, (waves_all + waves - 1) / waves), block(waves * TK_WAVE);
#define SS_CASE(NQ, PF) hipLaunchKernelGGL((ss_scan_kernel<NQ, PF>), grid, block, 0, stream, a, rec, ld_rec, np)
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
