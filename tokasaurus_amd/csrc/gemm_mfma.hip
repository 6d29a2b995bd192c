// bfloat16 matrix products for few rows (decode):  C[M,N] = A[M,K] * W[N,K]^T, M <= 128,
// on the gfx950 matrix cores with 32-bit accumulation, an optional RMSNorm of A fused
// in front and an epilogue fused behind.
//
// The product is bound by reading W once.  Weight rows are cut into tiles of 16;
// lane l of a wavefront streams the 8 values W[row l%16][32*step + 8*(l/16) .. +8]
// of a tile straight from memory into the first operand of v_mfma_f32_16x16x32_bf16
// (a row is read 64 contiguous bytes at a time); up to 16 tokens are the second
// operand, so
//     acc[j] of lane (r = l%16, q = l/16)  =  C[token 16*mb + r][row 16*tile + 4*q + j].
// No workgroup talks to another and partial sums inside a workgroup are added in
// wavefront order through LDS, so every output has one fixed order of summation.
//
// Two kernels (the entry point chooses; the engine calls it for up to 16 rows, for the
// stacked q, k, v product up to 32):
//   gemm_skinny_kernel: a workgroup owns NT tiles and all of K; its wavefronts split K
//     and read A straight from memory.
//   gemm_staged_kernel (a wide output, the head, from 5 rows on): a workgroup is
//     4 x WK wavefronts; the 4 wavefronts of a row own NT tiles each and share the K
//     range of their row, whose part of A passes through LDS (double buffered, 4 steps
//     of 32 a round) so that A is read from the caches once per workgroup and not once
//     per wavefront.
//
// Norm in front (sumsq_in != null).  The product of RMSNorm(x) is rstd[row] * ((x * w) W^T).
// The kernel that produced x (the residual epilogue below, when emit_w is given) has
// already written A = x * w, rounded once, and for every row the sum of x^2 over each
// of its tiles; this kernel adds those partial sums in tile order and scales its output
// rows by rstd = 1 / sqrt(sum / K + eps) in the epilogue.  So a norm between two
// products costs no kernel and no pass over the row of its own.
// A bias (one value an output, of the storage type) is added to the product in 32-bit before
// anything else happens to it.
// Epilogues: plain store, + residual (optionally emitting what the next norm needs),
// SwiGLU (the wavefront takes the same 16 rows of the gate and of the up projection),
// 32-bit store, and rotation with append: the output rows are [q heads | k heads |
// v heads]; a workgroup takes the rows (c, c + d/2) of a head together, rotates q and k
// by the token's position, writes q to the output and k and v into the token's page.
#include "common.h"

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8_t;
typedef __attribute__((ext_vector_type(4))) float f32x4_t;

enum { EPI_STORE = 0, EPI_RESIDUAL = 1, EPI_SWIGLU = 2, EPI_F32 = 3, EPI_ROPE = 4 };

struct GemmArgs {
  const bf16_t* A;
  int lda;
  const bf16_t* W;
  void* C;
  int ldc;
  const bf16_t* residual;
  int ldr;
  // norm in front: per row `parts_in` partial sums of squares of the un-normed row
  const float* sumsq_in;
  int parts_in;
  float eps;
  // residual epilogue, for the norm that follows: weight [N] (bfloat16, or float when
  // emit_w_f32), x * w rounded once [M, N], and per row one partial sum of x^2 a tile
  const void* emit_w;
  int emit_w_f32;
  bf16_t* emit_scaled;
  int ld_emit;
  float* emit_sumsq;
  int parts_out;
  // rotation with append
  const int* positions;
  const int* token_req;
  const int* block_table;
  int table_stride;
  const float* cos_t;  // [positions][d / 2], null: no rotation
  const float* sin_t;
  bf16_t* kcache;  // [page][kv head] pages of keys
  bf16_t* vcache;  // [page][kv head] pages of values
  int nq, nkv, d, P;
  const bf16_t* bias;  // [rows of W] or null: added to the product before the epilogue
  // the gated epilogue's other form (glu_limit > 0): g = min(gate, limit), u = clamp(up, -limit, limit),
  // g * sigmoid(glu_alpha * g) * (u + 1), 32-bit until the one rounding at the store
  float glu_limit, glu_alpha;
  int glu_gelu;  // the gated epilogue's third form: gelu(gate) * up with the tanh form of gelu
  float out_scale;  // the 32-bit epilogue multiplies its result by this (1: as it is)
  int M, N, K;  // N: outputs (for SwiGLU the intermediate size; W then has 2N rows, gate first)
  int TH;       // weight rows of a tile that are used (16, or 8 to make twice the workgroups of a narrow output)
};

// the bias of output `i` (a row of W), 0 without one; `i` is clamped to the rows there are
__device__ __forceinline__ float bias_at(const GemmArgs& a, int i, int rows) {
  return a.bias != nullptr ? __bfloat162float(a.bias[min(i, rows - 1)]) : 0.f;
}

template <int EPI>
__device__ __forceinline__ void store4(const GemmArgs& a, f32x4_t v, f32x4_t up, float scale, int token, int n) {
  if (token >= a.M) return;
  float o[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    o[j] = v[j] * scale + bias_at(a, n + j, a.N);
    if (EPI == EPI_SWIGLU) {
      const float g = v[j] * scale + bias_at(a, n + j, a.N), u = up[j] * scale + bias_at(a, a.N + n + j, 2 * a.N);
      if (a.glu_limit > 0.f) {
        o[j] = clamped_glu<bf16_t>(g, u, a.glu_limit, a.glu_alpha);
      } else if (a.glu_gelu) {
        const float gr = round_to<bf16_t>(g);
        o[j] = 0.5f * gr * (1.0f + tanhf(0.7978845608028654f * (gr + 0.044715f * gr * gr * gr))) * round_to<bf16_t>(u);
      } else {
        o[j] = silu_mul_bf16(g, u);
      }
    }
    if (EPI == EPI_RESIDUAL && n + j < a.N)
      o[j] = round_to<bf16_t>(o[j]) + __bfloat162float(a.residual[(size_t)token * a.ldr + n + j]);
  }
  if (EPI == EPI_F32) {
#pragma unroll
    for (int j = 0; j < 4; ++j) o[j] *= a.out_scale;
    float* c = (float*)a.C + (size_t)token * a.ldc + n;
    if (n + 3 < a.N && (a.ldc & 3) == 0) {
      *(f32x4_t*)c = f32x4_t{o[0], o[1], o[2], o[3]};
    } else {
#pragma unroll
      for (int j = 0; j < 4; ++j)
        if (n + j < a.N) c[j] = o[j];
    }
  } else {
    bf16_t* c = (bf16_t*)a.C + (size_t)token * a.ldc + n;
    if (n + 3 < a.N && (a.ldc & 3) == 0) {
      union { bf16_t h[4]; uint2 u; } pk;
#pragma unroll
      for (int j = 0; j < 4; ++j) pk.h[j] = __float2bfloat16(o[j]);
      *(uint2*)c = pk.u;
    } else {
#pragma unroll
      for (int j = 0; j < 4; ++j)
        if (n + j < a.N) c[j] = __float2bfloat16(o[j]);
    }
  }
}

__device__ __forceinline__ bf16x8_t zero8() {
  bf16x8_t z;
#pragma unroll
  for (int e = 0; e < 8; ++e) z[e] = (__bf16)0.f;
  return z;
}

// 1 / rms of every row of A from the partial sums its producer left, into LDS `scale`
// (16 * MB floats).  A wavefront takes a row at a time: every lane adds 4 parts (one
// 16-byte load), then the lanes' sums are added by a butterfly, so the order is fixed.
template <int MB>
__device__ __forceinline__ void row_scales(const GemmArgs& a, float* scale) {
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int nwaves = blockDim.x >> 6;
  const int rows = min(a.M, 16 * MB);
  const bool vec = (a.parts_in & 3) == 0;
  for (int token = wave; token < rows; token += nwaves) {
    const float* part = a.sumsq_in + (size_t)token * a.parts_in;
    float ss = 0.f;
    for (int p = lane * 4; p < a.parts_in; p += 256) {
      if (vec) {
        const f32x4_t v = *(const f32x4_t*)(part + p);
        ss += (v[0] + v[1]) + (v[2] + v[3]);
      } else {
        for (int j = 0; j < 4 && p + j < a.parts_in; ++j) ss += part[p + j];
      }
    }
    ss = wave_sum(ss);
    if (lane == 0) scale[token] = 1.0f / sqrtf(ss / (float)a.K + a.eps);
  }
}

// The residual epilogue's extra outputs for the norm that follows: x * w rounded once,
// and the sum of x^2 over this tile's columns.  All 64 lanes of a wavefront call this
// together; lanes (token, qq = 0..3) share a token.
__device__ __forceinline__ void emit_for_norm(const GemmArgs& a, const float (&x)[4], bool live, int token,
                                              int n, int part, int lane) {
  float ss = 0.f;
  if (live) {
    bf16_t* dst = a.emit_scaled + (size_t)token * a.ld_emit + n;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      if (n + j < a.N) {
        const float xr = round_to<bf16_t>(x[j]);
        const float w = a.emit_w_f32 ? ((const float*)a.emit_w)[n + j] : __bfloat162float(((const bf16_t*)a.emit_w)[n + j]);
        ss = fmaf(xr, xr, ss);
        dst[j] = __float2bfloat16(w * xr);
      }
    }
  }
  const float s1 = __shfl_xor(ss, 16, 64);
  const float lo = (lane & 16) ? s1 + ss : ss + s1;
  const float s2 = __shfl_xor(lo, 32, 64);
  const float total = (lane & 32) ? s2 + lo : lo + s2;
  if (live && (lane >> 4) == 0) a.emit_sumsq[(size_t)token * a.parts_out + part] = total;
}

// Rotation with append for 4 columns c .. c+3 of head h (and their partners c + d/2): x1, x2
// are the products rounded to bfloat16 as a plain store would leave them.
// What the rotation of one unit (token, head h, columns c .. c+3) reads besides the products;
// asked for before the main loop so that the epilogue does not wait for it.
struct RopeOperands {
  int pos, page;
  float cs[4], sn[4];
};

__device__ __forceinline__ RopeOperands rope_operands(const GemmArgs& a, int token, int h, int c) {
  RopeOperands r;
  const int half = a.d >> 1;
  const int t = min(token, a.M - 1);
  r.pos = a.positions[t];
  r.page = h >= a.nq ? a.block_table[(size_t)a.token_req[t] * a.table_stride + r.pos / a.P] : 0;
  const bool rotate = h < a.nq + a.nkv && a.cos_t != nullptr;
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const bool on = rotate && c + j < half;
    r.cs[j] = on ? a.cos_t[(size_t)r.pos * half + c + j] : 1.f;
    r.sn[j] = on ? a.sin_t[(size_t)r.pos * half + c + j] : 0.f;
  }
  return r;
}

__device__ __forceinline__ void rope_store(const GemmArgs& a, f32x4_t s0, f32x4_t s1, int token, int h, int c,
                                           const RopeOperands& r) {
  if (token >= a.M) return;
  const int half = a.d >> 1;
  const int pos = r.pos;
  float o1[4], o2[4];
  const bool rotate = h < a.nq + a.nkv && a.cos_t != nullptr;
  const int rows = (a.nq + 2 * a.nkv) * a.d;
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const float x1 = round_to<bf16_t>(s0[j] + bias_at(a, h * a.d + c + j, rows));
    const float x2 = round_to<bf16_t>(s1[j] + bias_at(a, h * a.d + c + j + half, rows));
    if (rotate && c + j < half) {
      rotate_pair(x1, x2, r.cs[j], r.sn[j], o1[j], o2[j]);
    } else {
      o1[j] = x1;
      o2[j] = x2;
    }
  }
  if (h < a.nq) {
    bf16_t* dst = (bf16_t*)a.C + (size_t)token * a.ldc + (size_t)h * a.d + c;
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (c + j < half) {
        dst[j] = __float2bfloat16(o1[j]);
        dst[j + half] = __float2bfloat16(o2[j]);
      }
    return;
  }
  const int page = r.page;
  const int off = pos % a.P;
  if (h < a.nq + a.nkv) {
    bf16_t* dst = a.kcache + ((size_t)page * a.nkv + (h - a.nq)) * a.P * a.d;
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (c + j < half) {
        dst[key_offset(a.P, off, c + j)] = __float2bfloat16(o1[j]);
        dst[key_offset(a.P, off, c + j + half)] = __float2bfloat16(o2[j]);
      }
  } else {
    bf16_t* dst = a.vcache + ((size_t)page * a.nkv + (h - a.nq - a.nkv)) * a.P * a.d;
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (c + j < half) {
        dst[value_offset(a.d, off, c + j)] = __float2bfloat16(o1[j]);
        dst[value_offset(a.d, off, c + j + half)] = __float2bfloat16(o2[j]);
      }
  }
}

#define SK_MAX_WAVES 16

// LDS of the skinny kernel: [scales: 16 * MB floats when NORM][sums: waves * NT * MB * 64 f32x4]
// FOLD (up to 8 rows of A, tiles of 8 weight rows, K a multiple of 64): a tile of 8 rows leaves
// half of the matrix core's 16 rows, and up to 8 rows of A half of its 16 columns, unused.  The
// upper 8 lanes of every 16 then take the same weight rows and the same rows of A over the second
// half of K: one product adds both halves' terms, into different quarters of the result (rows and
// columns 0..7: the first half of K, 8..15: the second; the other two quarters mix the halves and
// are not used), and the quarters are added when the wavefronts' sums are.  Every lane loads
// weights, and a wavefront issues half as many loads for the same bytes.
template <int MB, int NT, int EPI, bool NORM, bool FOLD = false>
__global__ __launch_bounds__(SK_MAX_WAVES * 64) void gemm_skinny_kernel(GemmArgs a) {
  extern __shared__ __align__(16) unsigned char smem[];
  constexpr int U = (NT + MB <= 3) ? 8 : ((NT + MB <= 6) ? 4 : 2);  // steps whose loads are in flight together
  constexpr bool PAIRED = EPI == EPI_SWIGLU || EPI == EPI_ROPE;     // two tiles that meet in the epilogue
  static_assert(!FOLD || (MB == 1 && NT == 1 && !PAIRED), "folding K takes one tile of 8 weight rows and up to 8 rows of A");
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int WK = blockDim.x >> 6;
  const int r = FOLD ? (lane & 7) : (lane & 15), q = lane >> 4;
  const int g = blockIdx.x;
  const int K32 = FOLD ? a.K >> 6 : (a.K + 31) >> 5;  // steps a lane walks (with FOLD: of its half of K)
  const size_t fold = FOLD ? (size_t)((lane >> 3) & 1) * (size_t)K32 * 32 : 0;  // where this lane's half of K begins
  const int ks0 = (int)((long)K32 * wave / WK), ks1 = (int)((long)K32 * (wave + 1) / WK);
  const bool k_exact = (a.K & 31) == 0;
  float* scales = (float*)smem;
  f32x4_t* red = (f32x4_t*)(smem + (NORM ? 16 * MB * sizeof(float) : 0));
  if (NORM) row_scales<MB>(a, scales);

  // rows of W this lane streams (clamped: rows past the end are masked at the store);
  // with tiles of 8 rows the upper lanes have no row and hold zeros
  const int TH = a.TH;
  const bool has_row = r < TH;  // (with FOLD: TH is 8 and r below it)
  int rope_head = 0, rope_col = 0;  // EPI_ROPE: the head and the first column of this workgroup's pair of tiles
  const bf16_t* wp[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t) {
    int row;
    if (EPI == EPI_SWIGLU) {
      row = min(g * TH + r, a.N - 1) + t * a.N;  // t = 0 gate, t = 1 up
    } else if (EPI == EPI_ROPE) {
      const int pairs = (a.d / 2 + TH - 1) / TH;  // pairs of tiles a head
      rope_head = g / pairs;
      rope_col = (g - rope_head * pairs) * TH;
      row = rope_head * a.d + min(rope_col + r, a.d / 2 - 1) + t * (a.d / 2);
    } else {
      row = min((g * NT + t) * TH + r, a.N - 1);
    }
    wp[t] = a.W + (size_t)row * a.K + q * 8 + fold;
  }
  const bf16_t* ap[MB];
#pragma unroll
  for (int mb = 0; mb < MB; ++mb) ap[mb] = a.A + (size_t)min(mb * 16 + r, a.M - 1) * a.lda + q * 8 + fold;

  // what the rotation of this thread's first unit reads besides the sums (position, page,
  // cos and sin) is asked for now, so that it has arrived when the main loop is through
  constexpr int UNITS = (PAIRED ? 1 : NT) * MB * 64;
  RopeOperands rope_pre = {};
  if (EPI == EPI_ROPE && tid < UNITS) {
    const int l0 = tid & 63, mb0 = (tid >> 6) % MB;
    rope_pre = rope_operands(a, mb0 * 16 + (l0 & 15), rope_head, rope_col + (l0 >> 4) * 4);
  }

  f32x4_t acc[NT][MB];
#pragma unroll
  for (int t = 0; t < NT; ++t)
#pragma unroll
    for (int mb = 0; mb < MB; ++mb) acc[t][mb] = f32x4_t{0.f, 0.f, 0.f, 0.f};

  int ks = ks0;
  if (k_exact) {
    for (; ks + U <= ks1; ks += U) {
      bf16x8_t w[U][NT], av[U][MB];
#pragma unroll
      for (int u = 0; u < U; ++u) {
#pragma unroll
        for (int t = 0; t < NT; ++t) {
          if (has_row) {
            w[u][t] = *(const bf16x8_t*)(wp[t] + (size_t)(ks + u) * 32);
          } else {
            w[u][t] = zero8();
          }
        }
#pragma unroll
        for (int mb = 0; mb < MB; ++mb) av[u][mb] = *(const bf16x8_t*)(ap[mb] + (size_t)(ks + u) * 32);
      }
#pragma unroll
      for (int u = 0; u < U; ++u)
#pragma unroll
        for (int t = 0; t < NT; ++t)
#pragma unroll
          for (int mb = 0; mb < MB; ++mb)
            acc[t][mb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(w[u][t], av[u][mb], acc[t][mb], 0, 0, 0);
    }
  }
  for (; ks < ks1; ++ks) {
    // a step may reach past K (K is a multiple of 8): read a valid chunk and zero the weight
    const bool k_ok = ks * 32 + q * 8 < a.K;
    const long off = k_ok ? (long)ks * 32 : -(long)(q * 8);
    bf16x8_t w[NT], av[MB];
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      w[t] = *(const bf16x8_t*)(wp[t] + off);
      if (!k_ok || !has_row) w[t] = zero8();
    }
#pragma unroll
    for (int mb = 0; mb < MB; ++mb) av[mb] = *(const bf16x8_t*)(ap[mb] + off);
#pragma unroll
    for (int t = 0; t < NT; ++t)
#pragma unroll
      for (int mb = 0; mb < MB; ++mb)
        acc[t][mb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(w[t], av[mb], acc[t][mb], 0, 0, 0);
  }

  // add the wavefronts' partial sums in wavefront order (with FOLD: the first half of K, then the second)
  if (WK > 1 || FOLD) {
#pragma unroll
    for (int t = 0; t < NT; ++t)
#pragma unroll
      for (int mb = 0; mb < MB; ++mb) red[(wave * NT * MB + t * MB + mb) * 64 + lane] = acc[t][mb];
  }
  if (WK > 1 || NORM || FOLD) __syncthreads();
  for (int u = tid; u < UNITS; u += blockDim.x) {
    const int l = u & 63, mb = (u >> 6) % MB, t = (u >> 6) / MB;
    const int token = mb * 16 + (l & 15), qq = l >> 4;
    f32x4_t s0 = f32x4_t{0.f, 0.f, 0.f, 0.f}, s1 = s0;
    if (FOLD) {
      // the second half's sums of (token, rows 4 qq ..) lie 8 tokens and 8 rows on: 8 + 2 * 16 lanes
      if (token < 8 && qq < 2) {
        for (int w = 0; w < WK; ++w) s0 += red[w * 64 + l];
        for (int w = 0; w < WK; ++w) s0 += red[w * 64 + l + 40];
      }
    } else if (WK > 1) {
      for (int w = 0; w < WK; ++w) {
        s0 += red[(w * NT * MB + t * MB + mb) * 64 + l];
        if (PAIRED) s1 += red[(w * NT * MB + MB + mb) * 64 + l];
      }
    } else {
      // one wavefront: unit u is this very lane's accumulator (u < 64 * NT * MB, tid == lane)
#pragma unroll
      for (int tt = 0; tt < NT; ++tt)
#pragma unroll
        for (int mm = 0; mm < MB; ++mm) {
          if (tt == t && mm == mb) s0 = acc[tt][mm];
          if (PAIRED && tt == 1 && mm == mb) s1 = acc[tt][mm];
        }
    }
    const float scale = NORM ? scales[token] : 1.0f;
    const bool live = qq * 4 < TH && token < a.M;  // (with FOLD: M is 8 at most)
    if (EPI == EPI_ROPE) {
      if (live)
        rope_store(a, s0 * scale, s1 * scale, token, rope_head, rope_col + qq * 4,
                   u == tid ? rope_pre : rope_operands(a, token, rope_head, rope_col + qq * 4));
    } else {
      const int tile = PAIRED ? g : g * NT + t;
      const int n = tile * TH + qq * 4;
      if (EPI == EPI_RESIDUAL && a.emit_w != nullptr) {
        float x[4];
#pragma unroll
        for (int j = 0; j < 4; ++j)
          x[j] = (live && n + j < a.N)
                     ? round_to<bf16_t>(s0[j] * scale + bias_at(a, n + j, a.N)) +
                           __bfloat162float(a.residual[(size_t)token * a.ldr + n + j])
                     : 0.f;
        emit_for_norm(a, x, live && n < a.N, token, n, tile, l);
      }
      if (live) store4<EPI>(a, s0, s1, scale, token, n);
    }
  }
}

// ---------------------------------------------------------------------------------
// 16 < M <= 128 (and any M for a wide output): A passes through LDS.
// A workgroup is 4 x WK wavefronts; wavefront (wn, wk) owns the NT tiles of index
// (4 * workgroup + wn) * NT + t and the steps of K that row wk of the workgroup has.
// A round is 4 steps; wavefront wn of a row brings step wn of the round into LDS in
// the lane order of the matrix-core operand (one KB a unit), for all MB blocks of 16
// tokens, while the round before is multiplied.
// LDS: [scales: 16 * MB floats when NORM][2 buffers x WK x 4 steps x MB units of 1 KB],
// the sums of the wavefront rows reuse the buffers after the last round.
// ---------------------------------------------------------------------------------
#define ST_WN 4
#define ST_SC 4

template <int MB, int NT, int EPI, bool NORM>
__global__ __launch_bounds__(1024) void gemm_staged_kernel(GemmArgs a) {
  extern __shared__ __align__(16) unsigned char smem[];
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int nwaves = blockDim.x >> 6;
  const int WK = nwaves / ST_WN;
  const int wn = wave % ST_WN, wk = wave / ST_WN;
  const int r = lane & 15, q = lane >> 4;
  const int K32 = (a.K + 31) >> 5;
  const int ks0 = (int)((long)K32 * wk / WK), ks1 = (int)((long)K32 * (wk + 1) / WK);
  const int rounds = ((K32 + WK - 1) / WK + ST_SC - 1) / ST_SC;
  float* scales = (float*)smem;
  unsigned char* stage = smem + (NORM ? 16 * MB * sizeof(float) : 0);
  bf16x8_t* stage_v = (bf16x8_t*)stage;  // [buffer][wk][step][mb][lane]
  f32x4_t* red = (f32x4_t*)stage;         // [wk][wn][NT * MB][lane], after the last round
  if (NORM) row_scales<MB>(a, scales);

  const int unit = blockIdx.x * ST_WN + wn;  // SwiGLU: a pair of tiles; else NT tiles
  const bf16_t* wp[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t) {
    int row;
    if (EPI == EPI_SWIGLU) {
      row = min(unit * 16 + r, a.N - 1) + t * a.N;
    } else {
      row = min((unit * NT + t) * 16 + r, a.N - 1);
    }
    wp[t] = a.W + (size_t)row * a.K + q * 8;
  }
  const bf16_t* ap[MB];
#pragma unroll
  for (int mb = 0; mb < MB; ++mb) ap[mb] = a.A + (size_t)min(mb * 16 + r, a.M - 1) * a.lda + q * 8;

  // this wavefront's step of a round of A, for every block of tokens
  auto load_a = [&](int round, bf16x8_t (&piece)[MB]) {
    const int s = ks0 + round * ST_SC + wn;
    const bool ok = s < ks1 && s * 32 + q * 8 < a.K;
#pragma unroll
    for (int mb = 0; mb < MB; ++mb) {
      if (ok) {
        piece[mb] = *(const bf16x8_t*)(ap[mb] + (size_t)s * 32);
      } else {
        piece[mb] = zero8();
      }
    }
  };
  auto store_a = [&](int buf, const bf16x8_t (&piece)[MB]) {
#pragma unroll
    for (int mb = 0; mb < MB; ++mb)
      stage_v[((((size_t)buf * WK + wk) * ST_SC + wn) * MB + mb) * 64 + lane] = piece[mb];
  };
  auto load_w = [&](int round, bf16x8_t (&w)[ST_SC][NT]) {
#pragma unroll
    for (int j = 0; j < ST_SC; ++j) {
      const int s = ks0 + round * ST_SC + j;
      const bool ok = s < ks1 && s * 32 + q * 8 < a.K;
#pragma unroll
      for (int t = 0; t < NT; ++t) {
        if (ok) {
          w[j][t] = *(const bf16x8_t*)(wp[t] + (size_t)s * 32);
        } else {
          w[j][t] = zero8();
        }
      }
    }
  };

  f32x4_t acc[NT][MB];
#pragma unroll
  for (int t = 0; t < NT; ++t)
#pragma unroll
    for (int mb = 0; mb < MB; ++mb) acc[t][mb] = f32x4_t{0.f, 0.f, 0.f, 0.f};

  bf16x8_t w_cur[ST_SC][NT], piece[MB];
  load_w(0, w_cur);
  load_a(0, piece);
  store_a(0, piece);
  __syncthreads();
  int buf = 0;
  for (int round = 0; round < rounds; ++round) {
    bf16x8_t w_nxt[ST_SC][NT];
    const bool more = round + 1 < rounds;
    if (more) {
      load_w(round + 1, w_nxt);
      load_a(round + 1, piece);
    }
#pragma unroll
    for (int j = 0; j < ST_SC; ++j) {
      // steps past this row's range carry zero weights: their product adds nothing
#pragma unroll
      for (int mb = 0; mb < MB; ++mb) {
        const bf16x8_t av = stage_v[((((size_t)buf * WK + wk) * ST_SC + j) * MB + mb) * 64 + lane];
#pragma unroll
        for (int t = 0; t < NT; ++t)
          acc[t][mb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(w_cur[j][t], av, acc[t][mb], 0, 0, 0);
      }
    }
    if (more) {
      store_a(buf ^ 1, piece);
#pragma unroll
      for (int j = 0; j < ST_SC; ++j)
#pragma unroll
        for (int t = 0; t < NT; ++t) w_cur[j][t] = w_nxt[j][t];
    }
    __syncthreads();
    buf ^= 1;
  }

  // add the rows' partial sums in row order
  constexpr int TN = (EPI == EPI_SWIGLU ? 1 : NT);
  if (WK == 1) {
    // every wavefront stores its own sums
    const int token0 = lane & 15, qq = lane >> 4;
#pragma unroll
    for (int mb = 0; mb < MB; ++mb) {
      const float scale = NORM ? scales[mb * 16 + token0] : 1.0f;
#pragma unroll
      for (int t = 0; t < TN; ++t) {
        const int n = (EPI == EPI_SWIGLU ? unit : unit * NT + t) * 16 + qq * 4;
        store4<EPI>(a, acc[t][mb], acc[NT - 1][mb], scale, mb * 16 + token0, n);
      }
    }
    return;
  }
#pragma unroll
  for (int t = 0; t < NT; ++t)
#pragma unroll
    for (int mb = 0; mb < MB; ++mb) red[((size_t)(wk * ST_WN + wn) * NT * MB + t * MB + mb) * 64 + lane] = acc[t][mb];
  __syncthreads();
  constexpr int UNITS = ST_WN * TN * MB * 64;
  for (int u = tid; u < UNITS; u += blockDim.x) {
    const int l = u & 63;
    int rest = u >> 6;
    const int mb = rest % MB;
    rest /= MB;
    const int t = rest % TN, own = rest / TN;
    const int token = mb * 16 + (l & 15), qq = l >> 4;
    f32x4_t s0 = f32x4_t{0.f, 0.f, 0.f, 0.f}, s1 = s0;
    for (int w = 0; w < WK; ++w) {
      s0 += red[((size_t)(w * ST_WN + own) * NT * MB + t * MB + mb) * 64 + l];
      if (EPI == EPI_SWIGLU) s1 += red[((size_t)(w * ST_WN + own) * NT * MB + MB + mb) * 64 + l];
    }
    const float scale = NORM ? scales[token] : 1.0f;
    const int tile_group = blockIdx.x * ST_WN + own;
    const int n = (EPI == EPI_SWIGLU ? tile_group : tile_group * NT + t) * 16 + qq * 4;
    store4<EPI>(a, s0, s1, scale, token, n);
  }
}

// ---------------------------------------------------------------------------------
// launch
// ---------------------------------------------------------------------------------
template <typename Kernel>
static bool allow_lds(Kernel kernel, size_t lds) {
  if (lds <= 64 * 1024) return true;
  return hipFuncSetAttribute((const void*)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds) == hipSuccess;
}

template <int MB, int NT, int EPI, bool NORM, bool FOLD = false>
static bool launch_skinny_one(const GemmArgs& a, int groups, int WK, hipStream_t stream) {
  size_t lds = (WK > 1 || FOLD) ? (size_t)WK * NT * MB * 64 * sizeof(f32x4_t) : 0;
  if (NORM) lds += (size_t)16 * MB * sizeof(float);
  auto kernel = gemm_skinny_kernel<MB, NT, EPI, NORM, FOLD>;
  if (!allow_lds(kernel, lds)) return false;
  hipLaunchKernelGGL(kernel, dim3(groups), dim3(WK * 64), lds, stream, a);
  return true;
}

// the skinny kernel with K folded into the unused half of the matrix core (one tile of 8 weight
// rows a workgroup, up to 8 rows of A)
static bool launch_folded(const GemmArgs& a, int epi, bool norm, int groups, int WK, hipStream_t stream) {
  switch (epi) {
    case EPI_RESIDUAL: return norm ? false : launch_skinny_one<1, 1, EPI_RESIDUAL, false, true>(a, groups, WK, stream);
    case EPI_STORE:
      return norm ? launch_skinny_one<1, 1, EPI_STORE, true, true>(a, groups, WK, stream)
                  : launch_skinny_one<1, 1, EPI_STORE, false, true>(a, groups, WK, stream);
    case EPI_F32:
      return norm ? launch_skinny_one<1, 1, EPI_F32, true, true>(a, groups, WK, stream)
                  : launch_skinny_one<1, 1, EPI_F32, false, true>(a, groups, WK, stream);
    default: return false;
  }
}

template <int MB, int NT, int EPI, bool NORM>
static bool launch_staged_one(const GemmArgs& a, int groups, int WK, hipStream_t stream) {
  size_t lds = (size_t)2 * WK * ST_SC * MB * 1024;
  const size_t red = WK > 1 ? (size_t)WK * ST_WN * NT * MB * 64 * sizeof(f32x4_t) : 0;
  if (red > lds) lds = red;
  if (NORM) lds += (size_t)16 * MB * sizeof(float);
  auto kernel = gemm_staged_kernel<MB, NT, EPI, NORM>;
  if (!allow_lds(kernel, lds)) return false;
  hipLaunchKernelGGL(kernel, dim3(groups), dim3(WK * ST_WN * 64), lds, stream, a);
  return true;
}

// the combinations that exist: a residual never follows a norm (the norm's product feeds a
// mixer or a feed-forward first), the staged kernel has neither rotation nor residual
template <int MB, bool STAGED>
static bool launch_mb(const GemmArgs& a, int epi, bool norm, int NT, int groups, int WK, hipStream_t stream) {
#define TK_ONE(NTV, E, NV) \
  (STAGED ? launch_staged_one<MB, NTV, (E == EPI_ROPE || E == EPI_RESIDUAL) ? EPI_STORE : E, NV>(a, groups, WK, stream) \
          : launch_skinny_one<MB, NTV, E, NV>(a, groups, WK, stream))
  switch (epi) {
    case EPI_SWIGLU: return norm ? TK_ONE(2, EPI_SWIGLU, true) : TK_ONE(2, EPI_SWIGLU, false);
    case EPI_ROPE: return STAGED ? false : (norm ? TK_ONE(2, EPI_ROPE, true) : TK_ONE(2, EPI_ROPE, false));
    case EPI_RESIDUAL: return (STAGED || norm) ? false : (NT == 1 ? TK_ONE(1, EPI_RESIDUAL, false) : TK_ONE(2, EPI_RESIDUAL, false));
    case EPI_STORE:
      if (NT == 1) return norm ? TK_ONE(1, EPI_STORE, true) : TK_ONE(1, EPI_STORE, false);
      return norm ? TK_ONE(2, EPI_STORE, true) : TK_ONE(2, EPI_STORE, false);
    case EPI_F32:
      if (NT == 1) return norm ? TK_ONE(1, EPI_F32, true) : TK_ONE(1, EPI_F32, false);
      return norm ? TK_ONE(2, EPI_F32, true) : TK_ONE(2, EPI_F32, false);
    default: return false;
  }
#undef TK_ONE
}

struct GemmExtra {
  // norm in front
  const float* sumsq_in;
  int parts_in;
  float eps;
  // residual epilogue: for the norm that follows
  const void* emit_w;
  int emit_w_f32;
  void* emit_scaled;
  int ld_emit;
  float* emit_sumsq;
  int parts_out;
  // rotation with append
  const int* positions;
  const int* token_req;
  const int* block_table;
  int table_stride;
  const float* cos_t;
  const float* sin_t;
  void* kcache;
  void* vcache;
  int nq, nkv, d, P;
  // a bias, one value a row of W, of the storage type
  const void* bias;
  // the gated epilogue with clamps (see GemmArgs); 0: the plain one
  float glu_limit, glu_alpha;
  // a factor on the 32-bit epilogue's result; 0 stands for none
  float out_scale;
  // the gated epilogue as gelu(gate) * up (tanh form); 0: not
  int glu_gelu;
};

// Number of partial sums a row gets from the residual epilogue with emit_w: one a tile.
// Compute units of the current device (the workgroups that run at a time, one each).
static int compute_units() {
  static int units = 0;
  if (units == 0) {
    int dev = 0, n = 0;
    if (hipGetDevice(&dev) == hipSuccess &&
        hipDeviceGetAttribute(&n, hipDeviceAttributeMultiprocessorCount, dev) == hipSuccess && n > 0)
      units = n;
    else
      units = 256;
  }
  return units;
}

// Weight rows of a tile that the skinny kernel uses for up to 32 rows of A: 16 fill the matrix
// core, fewer make more workgroups.  A workgroup streams its rows over all of K, so the time is
// that of the rounds of workgroups the compute units take, times the rows of each: the fewest
// win, and among equals the larger tile (A is read once a workgroup).  With two rounds or more
// of full tiles the rounds overlap and even out: 16 rows then (measured: smaller tiles lose).
// With the rotation epilogue (heads > 0) a workgroup takes `th` columns of one half of a head.
static int choose_tile_rows(int M, int N, int heads = 0, int half = 0) {
  if (M > 32) return 16;
  const int units = compute_units();
  int best = 16, best_cost = 0;
  for (int th = 16; th >= 8; th -= 4) {
    const int groups = heads > 0 ? heads * ((half + th - 1) / th) : (N + th - 1) / th;
    if (th == 16 && groups >= 2 * units) return 16;
    const int cost = ((groups + units - 1) / units) * th;
    if (th == 16 || cost < best_cost) { best = th; best_cost = cost; }
  }
  return best;
}

TK_API int tk_gemm_skinny_parts(int M, int N, int tile_rows) {
  const int th = tile_rows > 0 ? tile_rows : choose_tile_rows(M, N);
  return (N + th - 1) / th;
}

// A [M, K] bfloat16 (rows lda apart), W [N, K] row-major ([2N, K] gate over up for SwiGLU),
// C [M, N] ([M, nq * d] with the rotation epilogue).  `extra` (may be null) carries the
// norm in front, the outputs for a following norm and the rotation's operands.
// waves_k: wavefronts (skinny) or wavefront rows (staged) that split K inside a workgroup
// (0 = choose); tiles: weight tiles per wavefront, 1 or 2 (0 = choose; SwiGLU and the rotation
// always pair); staged: -1 = choose, 0 = skinny, 1 = staged; tile_rows: weight rows of a
// tile that the skinny kernel uses, 16 or 8 (0 = choose; tk_gemm_skinny_parts tells the
// choice to whoever sizes emit_sumsq); fold: 0 = never fold K into the unused half of the matrix
// core, else where it can be done (tiles of 8 weight rows, up to 8 rows of A: gemm_skinny_kernel).
TK_API int tk_gemm_skinny_bf16(const void* A, int lda, const void* W, void* C, int ldc,
                               const void* residual, int ldr, const GemmExtra* extra, int M, int N,
                               int K, int epi, int waves_k, int tiles, int staged, int tile_rows, int fold,
                               hipStream_t stream) {
  TK_REQUIRE(M >= 0 && N > 0 && K > 0, "gemm_skinny: bad sizes M=%d N=%d K=%d", M, N, K);
  TK_REQUIRE(M <= 128, "gemm_skinny: at most 128 rows, got %d", M);
  TK_REQUIRE(epi >= EPI_STORE && epi <= EPI_ROPE, "gemm_skinny: unknown epilogue %d", epi);
  TK_REQUIRE(K % 8 == 0, "gemm_skinny: K=%d must be a multiple of 8 for the bfloat16 kernels", K);
  TK_REQUIRE(lda % 8 == 0 && ((uintptr_t)A & 15) == 0 && ((uintptr_t)W & 15) == 0,
             "gemm_skinny: rows of A and W must be 16-byte aligned (lda=%d)", lda);
  TK_REQUIRE(lda >= K, "gemm_skinny: lda %d shorter than K %d", lda, K);
  TK_REQUIRE(epi != EPI_RESIDUAL || (residual && ldr >= N), "gemm_skinny: residual missing or too narrow");
  TK_REQUIRE(tile_rows == 0 || tile_rows == 4 || tile_rows == 8 || tile_rows == 12 || tile_rows == 16, "gemm_skinny: tile_rows %d is not 0, 4, 8, 12 or 16", tile_rows);
  if (M == 0) return 0;
  GemmArgs a = {};
  a.A = (const bf16_t*)A; a.lda = lda; a.W = (const bf16_t*)W; a.C = C; a.ldc = ldc;
  a.residual = (const bf16_t*)residual; a.ldr = ldr; a.M = M; a.N = N; a.K = K; a.TH = 16;
  a.out_scale = 1.f;
  bool norm = false;
  if (extra) {
    a.sumsq_in = extra->sumsq_in; a.parts_in = extra->parts_in; a.eps = extra->eps;
    a.emit_w = extra->emit_w; a.emit_w_f32 = extra->emit_w_f32; a.emit_scaled = (bf16_t*)extra->emit_scaled;
    a.ld_emit = extra->ld_emit; a.emit_sumsq = extra->emit_sumsq; a.parts_out = extra->parts_out;
    a.positions = extra->positions; a.token_req = extra->token_req; a.block_table = extra->block_table;
    a.table_stride = extra->table_stride; a.cos_t = extra->cos_t; a.sin_t = extra->sin_t;
    a.kcache = (bf16_t*)extra->kcache; a.vcache = (bf16_t*)extra->vcache;
    a.nq = extra->nq; a.nkv = extra->nkv; a.d = extra->d; a.P = extra->P;
    a.bias = (const bf16_t*)extra->bias;
    a.glu_limit = extra->glu_limit; a.glu_alpha = extra->glu_alpha; a.glu_gelu = extra->glu_gelu;
    if (extra->out_scale != 0.f) a.out_scale = extra->out_scale;
    norm = a.sumsq_in != nullptr;
  }
  TK_REQUIRE(!norm || a.parts_in > 0, "gemm_skinny: a norm in front needs its partial sums");
  TK_REQUIRE(!(norm && epi == EPI_RESIDUAL), "gemm_skinny: a norm in front cannot be combined with a residual behind");
  TK_REQUIRE(a.emit_w == nullptr || (epi == EPI_RESIDUAL && a.emit_scaled && a.emit_sumsq && a.ld_emit >= N),
             "gemm_skinny: outputs for a following norm go with the residual epilogue and need their buffers");
  if (epi == EPI_ROPE) {
    TK_REQUIRE(extra && a.positions && a.token_req && a.block_table && a.kcache && a.vcache,
               "gemm_skinny: the rotation epilogue needs positions, the block table and the cache");
    TK_REQUIRE(a.nq > 0 && a.nkv > 0 && a.d > 0 && a.d % 8 == 0 && a.P > 0 && N == (a.nq + 2 * a.nkv) * a.d,
               "gemm_skinny: rotation epilogue with nq=%d nkv=%d d=%d does not match N=%d", a.nq, a.nkv, a.d, N);
    TK_REQUIRE((a.cos_t == nullptr) == (a.sin_t == nullptr), "gemm_skinny: cos and sin tables go together");
    TK_REQUIRE(ldc >= a.nq * a.d, "gemm_skinny: ldc %d shorter than the query heads", ldc);
  } else {
    TK_REQUIRE(ldc >= N, "gemm_skinny: ldc %d shorter than N %d", ldc, N);
  }

  const int n16 = (N + 15) / 16;
  const int MB = M <= 16 ? 1 : (M <= 32 ? 2 : (M <= 64 ? 4 : 8));
  const int K32 = (K + 31) / 32;
  // measured on an MI355X: passing A through LDS pays for a wide output (the head) from 5 rows on,
  // where many wavefronts of a workgroup share it; a narrow one needs every tile in a workgroup of its own
  const bool can_stage = epi != EPI_ROPE && epi != EPI_RESIDUAL;
  const bool use_staged = can_stage && (staged < 0 ? M > 4 && K32 >= 2 * ST_SC && n16 >= 2048 : staged != 0);
  const bool paired = epi == EPI_SWIGLU || epi == EPI_ROPE;
  int NT = paired ? 2 : (tiles > 0 ? tiles : 1);
  TK_REQUIRE(NT == 1 || NT == 2, "gemm_skinny: tiles=%d outside 1..2", NT);
  bool ok;
  if (use_staged) {
    const int units = paired ? n16 : (n16 + NT - 1) / NT;  // what one wavefront row owns
    const int groups = (units + ST_WN - 1) / ST_WN;
    int WK = waves_k;
    if (WK <= 0) {
      WK = (1024 + groups * ST_WN - 1) / (groups * ST_WN);  // about a thousand wavefronts
      if (WK < 2) WK = 2;                                   // two rows a workgroup measured best
    }
    const int lds_cap = (128 * 1024) / (2 * ST_SC * MB * 1024);        // two buffers within 128 KB
    if (WK > lds_cap) WK = lds_cap;
    if (WK > K32 / ST_SC) WK = K32 / ST_SC;                            // at least a round each
    if (WK > 16 / ST_WN) WK = 16 / ST_WN;
    if (WK < 1) WK = 1;
    switch (MB) {
      case 1: ok = launch_mb<1, true>(a, epi, norm, NT, groups, WK, stream); break;
      case 2: ok = launch_mb<2, true>(a, epi, norm, NT, groups, WK, stream); break;
      case 4: ok = launch_mb<4, true>(a, epi, norm, NT, groups, WK, stream); break;
      default: ok = launch_mb<8, true>(a, epi, norm, NT, groups, WK, stream); break;
    }
  } else {
    a.TH = tile_rows > 0 ? tile_rows
                         : (epi == EPI_ROPE ? choose_tile_rows(M, N, a.nq + 2 * a.nkv, a.d / 2) : choose_tile_rows(M, N));
    const int th_units = (N + a.TH - 1) / a.TH;
    int groups;
    if (epi == EPI_ROPE) {
      groups = (a.nq + 2 * a.nkv) * ((a.d / 2 + a.TH - 1) / a.TH);
    } else {
      groups = paired ? th_units : (th_units + NT - 1) / NT;
    }
    TK_REQUIRE(a.emit_w == nullptr || a.parts_out == th_units, "gemm_skinny: %d partial sums a row, the caller sized for %d", th_units, a.parts_out);
    // tiles of 8 weight rows for up to 8 rows of A: both halves of K in one product
    const bool folded = fold != 0 && a.TH == 8 && M <= 8 && NT == 1 && !paired && K % 64 == 0 && !(norm && epi == EPI_RESIDUAL);
    const int steps = folded ? K32 / 2 : K32;  // steps of 32 that a lane walks
    int WK = waves_k;
    if (WK <= 0) {
      // a wavefront issues the loads of U steps together: best when that is all it has to do,
      // so that the whole matrix is asked for at once and the hardware queues the workgroups
      const int U = (NT + MB <= 3) ? 8 : ((NT + MB <= 6) ? 4 : 2);
      WK = steps / (U * NT);
    }
    const int lds_cap = 65536 / (NT * MB * 64 * (int)sizeof(f32x4_t));
    if (WK > lds_cap) WK = lds_cap;
    if (WK > SK_MAX_WAVES) WK = SK_MAX_WAVES;
    if (WK > steps) WK = steps;
    if (WK < 1) WK = 1;
    if (folded) {
      ok = launch_folded(a, epi, norm, groups, WK, stream);
    } else
    switch (MB) {
      case 1: ok = launch_mb<1, false>(a, epi, norm, NT, groups, WK, stream); break;
      case 2: ok = launch_mb<2, false>(a, epi, norm, NT, groups, WK, stream); break;
      case 4: ok = launch_mb<4, false>(a, epi, norm, NT, groups, WK, stream); break;
      default: ok = launch_mb<8, false>(a, epi, norm, NT, groups, WK, stream); break;
    }
  }
  TK_REQUIRE(ok, "gemm_skinny: no kernel for this combination, or its local memory could not be reserved");
  TK_CHECK_LAUNCH("gemm_skinny");
  return 0;
}
