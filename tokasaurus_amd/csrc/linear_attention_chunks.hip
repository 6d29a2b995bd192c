// Linear attention in chunks of 64 tokens as products on the matrix cores, for the forms whose decays are at most one and
// come with a portion's tokens: LA_CHANNEL and LA_MEMORY of linear_attention.hip, whose sums these are in another order.
// Every product is one of 32-bit numbers (v_mfma_f32_16x16x4_f32), in either storage type.
//
// Inside a chunk let A_t be the sum of the decays' logarithms from the chunk's first token to token t (a number per row of S,
// or in LA_MEMORY one for all rows), w_s the factor on what token s writes (1, or exp(i - m)), and S the state in front of it:
//     o_t = (exp(A_t) q_t)^T S + sum_{s <= t} P_ts v_s          P_ts = sum_i q_t,i k_s,i exp(A_t,i - A_s,i) w_s
//     S  <- exp(A_last) S + sum_s (exp(A_last - A_s) w_s k_s) v_s^T
// No exponent is positive as it stands, and none becomes so: P is computed in blocks of 16 x 16 tokens, off the diagonal as a
// product of q_t exp(A_t - R) and k_s exp(R - A_s) with R the sum in front of the block of t (s <= R's token < t).  On the
// diagonal the second exponent is positive; where it stays below LC_REACH in every channel (the decays of 16 tokens leave
// more than 2^-LC_REACH) both factors and their product are numbers as good as any, else the block is summed pair by pair.
//
// Two kernels.  The first works on all (chunk, head) at once: decays, their sums, and the factors of the products above, in
// `rec`.  The second walks a request's chunks for 16 columns of a head's state in a workgroup: per chunk two products on what
// the first has left and one update of S, which stays in registers and goes round through LDS.
#include "linear_attention.h"

typedef float v4f __attribute__((ext_vector_type(4)));

#define LC_CHUNK 64
#define LC_SLAB 64       // rows of S (key channels) that the first kernel works on at a time
#define LC_LD 68         // a row of a slab in LDS: 64 numbers and the padding that spreads rows over the banks
#define LC_RANK 16       // low-rank sums staged at a time
#define LC_MAX_SLABS 4   // key heads of up to 256 channels
#define LC_FROM 32       // tokens of a step's longest portion from which on it goes in chunks
#define LC_REACH 60.f
#define LC_LOG2E 1.44269504088896341f

__device__ __forceinline__ float lc_exp2(float x) { return __builtin_amdgcn_exp2f(x); }

// What a (chunk, head) leaves in `rec`: the factors of q and of k, P, and the decay of S over the chunk [dkp].  The first three
// lie as the lanes of the second kernel read them, 64 lanes' four numbers side by side: lane 16 c + col of block
//     q [w][m]   has token 16 w + col, channels 16 m + 4 c + e
//     k [n][T]   has channel 16 n + col, tokens 16 T + 4 c + e
//     P [w][T]   has token 16 w + col, tokens s = 16 T + 4 c + e
__host__ __device__ __forceinline__ size_t lc_words(int dkp) { return (size_t)2 * LC_CHUNK * dkp + LC_CHUNK * LC_CHUNK + dkp; }
__host__ __device__ __forceinline__ size_t lc_k_at(int dkp) { return (size_t)LC_CHUNK * dkp; }
__host__ __device__ __forceinline__ size_t lc_p_at(int dkp) { return (size_t)2 * LC_CHUNK * dkp; }
__host__ __device__ __forceinline__ size_t lc_d_at(int dkp) { return lc_p_at(dkp) + LC_CHUNK * LC_CHUNK; }

bool la_chunks_take(int mode, int dk, int longest) {
  return (mode == LA_CHANNEL || mode == LA_MEMORY) && dk <= LC_SLAB * LC_MAX_SLABS && longest >= LC_FROM;
}

// --------------------------------------------------------------------------
// The first kernel.  A workgroup a (chunk, head); wavefront g owns tokens 16 g .. 16 g + 15: as a channel a lane for loading and
// summing, as rows of a block of P for the products.  Tokens beyond the request's end have q = k = 0 and no decay.
// --------------------------------------------------------------------------
template <int MODE>
__global__ __launch_bounds__(256) void la_chunk_factors_kernel(LaArgs a, int dkp, const float* __restrict__ proj,
                                                               const float2* __restrict__ gates, float* __restrict__ rec) {
  constexpr bool CHANNEL = MODE == LA_CHANNEL;
  __shared__ __align__(16) float qs[LC_CHUNK * LC_LD], ks[LC_CHUNK * LC_LD], as[CHANNEL ? LC_CHUNK * LC_LD : LC_CHUNK];
  __shared__ __align__(16) float low[CHANNEL ? LC_RANK * LC_LD : 4], sums[CHANNEL ? 4 * LC_SLAB : 4], ws[CHANNEL ? 4 : LC_CHUNK];
  const int chunk = blockIdx.x, h = blockIdx.y;
  const int r = a.chunk_req[chunk], row0 = a.chunk_row0[chunk], last = a.q_start[r + 1];
  const int lane = threadIdx.x & (TK_WAVE - 1), g = __builtin_amdgcn_readfirstlane(threadIdx.x / TK_WAVE);
  const int col = lane & 15, c = lane >> 4;
  float* out = rec + ((size_t)chunk * a.H + h) * lc_words(dkp);
  const int t0 = row0 + 16 * g;
  if (!CHANNEL && g == 0) {
    const int t = row0 + lane;
    const float2 e = t < last ? gates[(size_t)t * a.H + h] : make_float2(0.f, 0.f);
    float l = e.x;
#pragma unroll
    for (int o = 1; o < LC_CHUNK; o <<= 1) {
      const float up = __shfl_up(l, o, TK_WAVE);
      if (lane >= o) l += up;
    }
    as[lane] = l * LC_LOG2E;
    ws[lane] = e.y;
  }
  v4f acc[4];
#pragma unroll
  for (int J = 0; J < 4; ++J) acc[J] = (v4f){0.f, 0.f, 0.f, 0.f};
  float diag[4] = {0.f, 0.f, 0.f, 0.f};  // (of diagonal blocks that are summed pair by pair)
  auto stage = [&](int r0, int nr) {  // the chunk's low-rank sums r0 .. r0 + nr - 1
    for (int i = threadIdx.x; i < LC_CHUNK * nr; i += 256) {
      const int t = i / nr, k = i % nr;
      low[k * LC_LD + t] = proj[(size_t)min(row0 + t, last - 1) * a.ld + a.low_off + r0 + k];
    }
  };
  if (CHANNEL) stage(0, min(LC_RANK, a.rank));
  __syncthreads();

  for (int n0 = 0; n0 < dkp; n0 += LC_SLAB) {
    const int ch = n0 + lane, x = h * a.dk + ch;
    const bool in = ch < a.dk;
    float A[16], qv[16], kv[16];
#pragma unroll
    for (int j = 0; j < 16; ++j) {
      const float* row = proj + (size_t)min(t0 + j, last - 1) * a.ld + (in ? x : 0);
      qv[j] = row[a.q_off];
      kv[j] = row[a.k_off];
    }
    bool near = true;  // the diagonal block goes as a product
    if (CHANNEL) {
      const int width = a.H * a.dk;
#pragma unroll
      for (int j = 0; j < 16; ++j) A[j] = 0.f;
      for (int r0 = 0; r0 < a.rank; r0 += LC_RANK) {
        const int nr = min(LC_RANK, a.rank - r0);
        float up[LC_RANK];
#pragma unroll
        for (int k = 0; k < LC_RANK; ++k) up[k] = in && k < nr ? a.low_up[(size_t)(r0 + k) * width + x] : 0.f;
        if (a.rank > LC_RANK) {
          __syncthreads();
          stage(r0, nr);
          __syncthreads();
        }
#pragma unroll
        for (int k = 0; k < LC_RANK; ++k) {
          if (k >= nr) break;
          const float4* lt = (const float4*)(low + k * LC_LD + 16 * g);
#pragma unroll
          for (int j = 0; j < 4; ++j) {
            const float4 l4 = lt[j];
            A[4 * j] = fmaf(l4.x, up[k], A[4 * j]); A[4 * j + 1] = fmaf(l4.y, up[k], A[4 * j + 1]);
            A[4 * j + 2] = fmaf(l4.z, up[k], A[4 * j + 2]); A[4 * j + 3] = fmaf(l4.w, up[k], A[4 * j + 3]);
          }
        }
      }
      const float bias = in ? a.low_bias[x] : 0.f;
      float sum = 0.f;
#pragma unroll
      for (int j = 0; j < 16; ++j) {
        sum += in && t0 + j < last ? la_log_sigmoid(A[j] + bias) / a.tau * LC_LOG2E : 0.f;
        A[j] = sum;
      }
      sums[g * LC_SLAB + lane] = sum;
      near = __all(sum > -LC_REACH);
    }
#pragma unroll
    for (int j = 0; j < 16; ++j) {
      const bool valid = in && t0 + j < last;
      qs[(16 * g + j) * LC_LD + lane] = valid ? qv[j] * a.q_scale : 0.f;
      kv[j] = valid ? kv[j] : 0.f;
      ks[(16 * g + j) * LC_LD + lane] = kv[j];
    }
    float end;
    if (CHANNEL) {
      __syncthreads();
      float before = 0.f;
      end = 0.f;
#pragma unroll
      for (int w = 0; w < 4; ++w) {
        const float s = sums[w * LC_SLAB + lane];
        if (w < g) before += s;
        end += s;
      }
#pragma unroll
      for (int j = 0; j < 16; ++j) {
        A[j] += before;
        as[(16 * g + j) * LC_LD + lane] = A[j];
      }
    } else {
      end = as[LC_CHUNK - 1];
#pragma unroll
      for (int j = 0; j < 16; ++j) {
        A[j] = as[16 * g + j];
        kv[j] *= ws[16 * g + j];
      }
    }
    // the factors of the products that the second kernel makes (those of q below)
    {
      float4* kt = (float4*)(out + lc_k_at(dkp)) + ((ch / 16) * 4 + g) * TK_WAVE + col;
#pragma unroll
      for (int j = 0; j < 4; ++j)
        kt[16 * j] = make_float4(kv[4 * j] * lc_exp2(end - A[4 * j]), kv[4 * j + 1] * lc_exp2(end - A[4 * j + 1]),
                            kv[4 * j + 2] * lc_exp2(end - A[4 * j + 2]), kv[4 * j + 3] * lc_exp2(end - A[4 * j + 3]));
    }
    if (g == 0) out[lc_d_at(dkp) + ch] = lc_exp2(end);
    __syncthreads();
    // rows 16 g .. of P, transposed: a lane has row 16 J + col of the first operand (k) and column 16 g + col of the second (q),
    // and of every 16 channels the four from 4 c on; it ends up with P of token 16 g + col and tokens s = 16 J + 4 c + i.
#pragma unroll
    for (int m = 0; m < LC_SLAB / 16; ++m) {
      const int at = 16 * m + 4 * c;
      float4 q4 = *(const float4*)(qs + (16 * g + col) * LC_LD + at);
      float4 a4, ref = make_float4(0.f, 0.f, 0.f, 0.f);
      if (CHANNEL) {
        a4 = *(const float4*)(as + (16 * g + col) * LC_LD + at);
      } else {
        const float l = as[16 * g + col];
        a4 = make_float4(l, l, l, l);
      }
      ((float4*)out)[(g * (dkp / 16) + n0 / 16 + m) * TK_WAVE + lane] =
          make_float4(q4.x * lc_exp2(a4.x), q4.y * lc_exp2(a4.y), q4.z * lc_exp2(a4.z), q4.w * lc_exp2(a4.w));
      if (CHANNEL) {
        if (g > 0) ref = *(const float4*)(as + (16 * g - 1) * LC_LD + at);
        q4.x *= lc_exp2(a4.x - ref.x); q4.y *= lc_exp2(a4.y - ref.y); q4.z *= lc_exp2(a4.z - ref.z); q4.w *= lc_exp2(a4.w - ref.w);
      }
#pragma unroll
      for (int J = 0; J < 4; ++J) {
        if (J > g || (J == g && !near)) continue;  // (the same for all lanes)
        float4 k4 = *(const float4*)(ks + (16 * J + col) * LC_LD + at);
        if (CHANNEL) {
          const float4 b4 = *(const float4*)(as + (16 * J + col) * LC_LD + at);
          k4.x *= lc_exp2(ref.x - b4.x); k4.y *= lc_exp2(ref.y - b4.y); k4.z *= lc_exp2(ref.z - b4.z); k4.w *= lc_exp2(ref.w - b4.w);
        }
        acc[J] = __builtin_amdgcn_mfma_f32_16x16x4f32(k4.x, q4.x, acc[J], 0, 0, 0);
        acc[J] = __builtin_amdgcn_mfma_f32_16x16x4f32(k4.y, q4.y, acc[J], 0, 0, 0);
        acc[J] = __builtin_amdgcn_mfma_f32_16x16x4f32(k4.z, q4.z, acc[J], 0, 0, 0);
        acc[J] = __builtin_amdgcn_mfma_f32_16x16x4f32(k4.w, q4.w, acc[J], 0, 0, 0);
      }
    }
    if (CHANNEL && !near) {
      // the block on the diagonal: the lane's four pairs (token 16 g + col, tokens s = 16 g + 4 c + i), as a product leaves them
#pragma unroll 4
      for (int m = 0; m < LC_SLAB / 4; ++m) {
        const float4 q4 = *(const float4*)(qs + (16 * g + col) * LC_LD + 4 * m), a4 = *(const float4*)(as + (16 * g + col) * LC_LD + 4 * m);
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const float4 k4 = *(const float4*)(ks + (16 * g + 4 * c + i) * LC_LD + 4 * m);
          const float4 b4 = *(const float4*)(as + (16 * g + 4 * c + i) * LC_LD + 4 * m);
          // (pairs with s behind the token are dropped below: their exponents are kept from overflowing)
          diag[i] = fmaf(q4.x * k4.x, lc_exp2(fminf(a4.x - b4.x, 0.f)), diag[i]);
          diag[i] = fmaf(q4.y * k4.y, lc_exp2(fminf(a4.y - b4.y, 0.f)), diag[i]);
          diag[i] = fmaf(q4.z * k4.z, lc_exp2(fminf(a4.z - b4.z, 0.f)), diag[i]);
          diag[i] = fmaf(q4.w * k4.w, lc_exp2(fminf(a4.w - b4.w, 0.f)), diag[i]);
        }
      }
    }
    __syncthreads();  // the slab is used up
  }
  // P as far as the second kernel uses it: up to the diagonal block's end
#pragma unroll
  for (int J = 0; J < 4; ++J) {
    if (J > g) continue;
    float p[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int t = 16 * g + col, s = 16 * J + 4 * c + i;
      p[i] = CHANNEL ? acc[J][i] + (J == g ? diag[i] : 0.f) : acc[J][i] * (lc_exp2(fminf(as[t] - as[s], 0.f)) * ws[s]);
      if (s > t) p[i] = 0.f;
    }
    ((float4*)(out + lc_p_at(dkp)))[(g * 4 + J) * TK_WAVE + lane] = make_float4(p[0], p[1], p[2], p[3]);
  }
}

// --------------------------------------------------------------------------
// The second kernel.  A workgroup owns 16 columns of the state of one (head, request): wavefront w computes the results of
// tokens 16 w .. of every chunk, and the rows 16 (w + 4 p) .. of S, whose tiles of 16 x 16 stay in its registers and are
// handed to the others through LDS, [row / 4][column][4], in two buffers.  What a chunk needs is asked for while the chunk
// before is computed, into one of two sets of registers in turn, and waited for once, in front of the chunk.  (P right of the
// block of the diagonal is read with the rest and not used.)  The loads stand between the products: issued together in front of
// them they would hold the products up.  NP: tiles of S of a wavefront (slabs of 64 rows).
// --------------------------------------------------------------------------
template <int NP>
struct LcChunk {
  float4 q[4 * NP], k[4 * NP], p[4], d[NP];
  float v[4];  // of tokens 16 w + 4 c + e: a wavefront brings a quarter of a chunk's values, which go round through LDS
};

template <int MODE, int NP>
__global__ __launch_bounds__(256) void la_chunk_walk_kernel(LaArgs a, const float* __restrict__ proj, const float* __restrict__ rec,
                                                            float* __restrict__ o) {
  constexpr int DKP = LC_SLAB * NP;
  __shared__ __align__(16) float s_lds[2][DKP * 16], v_lds[2][LC_CHUNK * 16];
  const int h = blockIdx.x, r = blockIdx.y;
  const int c0 = a.first_chunk[r], c1 = a.first_chunk[r + 1];
  if (c0 >= c1) return;
  const int first = a.q_start[r], last = a.q_start[r + 1];
  const int lane = threadIdx.x & (TK_WAVE - 1), w = __builtin_amdgcn_readfirstlane(threadIdx.x / TK_WAVE);
  const int col = lane & 15, c = lane >> 4;
  const int columns = la_columns<MODE>(a.dv), j = blockIdx.z * 16 + col;
  const bool live = j < columns;
  const bool one = MODE == LA_MEMORY && j == a.dv;  // the column that sums the keys
  const int v_at = a.v_off + h * a.dv + min(j, a.dv - 1);
  float* s_col = a.state + (size_t)a.slots[r] * a.state_stride + ((size_t)h * columns + (live ? j : 0)) * a.dk;
  v4f s[NP];
#pragma unroll
  for (int p = 0; p < NP; ++p)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int n = 16 * (w + 4 * p) + 4 * c + i;
      s[p][i] = live && n < a.dk ? s_col[n] : 0.f;
    }
  // The loads of a chunk, piece by piece: m < 4 NP (q and k), T < 4 (P, and with the first all else)
  auto ask_qk = [&](LcChunk<NP>& x, const float* src, int m) {
    x.q[m] = ((const float4*)src)[(w * (DKP / 16) + m) * TK_WAVE + lane];
    x.k[m] = ((const float4*)(src + lc_k_at(DKP)))[((w + 4 * (m / 4)) * 4 + m % 4) * TK_WAVE + lane];
  };
  auto ask_p = [&](LcChunk<NP>& x, const float* src, int chunk, int T) {
    x.p[T] = ((const float4*)(src + lc_p_at(DKP)))[(w * 4 + T) * TK_WAVE + lane];
    if (T == 0) {
#pragma unroll
      for (int p = 0; p < NP; ++p) x.d[p] = *(const float4*)(src + lc_d_at(DKP) + 16 * (w + 4 * p) + 4 * c);
      const int t0 = first + (chunk - c0) * LC_CHUNK + 16 * w + 4 * c;
#pragma unroll
      for (int e = 0; e < 4; ++e) x.v[e] = proj[(size_t)min(t0 + e, last - 1) * a.ld + v_at];
    }
  };
  auto left_by = [&](int chunk) { return rec + ((size_t)chunk * a.H + h) * lc_words(DKP); };
  // S, and the next chunk's values, to the other wavefronts
  auto hand = [&](const LcChunk<NP>& x, int buf) {
    *(float4*)(v_lds[buf] + (w * TK_WAVE + lane) * 4) = one ? make_float4(1.f, 1.f, 1.f, 1.f) : make_float4(x.v[0], x.v[1], x.v[2], x.v[3]);
#pragma unroll
    for (int p = 0; p < NP; ++p)
      *(float4*)(s_lds[buf] + ((4 * (w + 4 * p) + c) * 16 + col) * 4) = make_float4(s[p][0], s[p][1], s[p][2], s[p][3]);
  };
  // one chunk: the results of its tokens, the state behind it
  auto take = [&](const LcChunk<NP>& x, LcChunk<NP>& next, int chunk, int buf) {
    const int ahead = min(chunk + 1, c1 - 1);
    const float* src = left_by(ahead);
    // what the state in front of the chunk gives its tokens, and what the tokens give each other
    v4f y0 = (v4f){0.f, 0.f, 0.f, 0.f}, y1 = y0;
    float4 sm[4 * NP], vm[4];
#pragma unroll
    for (int T = 0; T < 4; ++T) vm[T] = *(const float4*)(v_lds[buf] + (T * TK_WAVE + lane) * 4);
#pragma unroll
    for (int m = 0; m < 4 * NP; ++m) sm[m] = *(const float4*)(s_lds[buf] + ((4 * m + c) * 16 + col) * 4);
    __builtin_amdgcn_sched_barrier(0);  // (all of them on their way before the first product)
#pragma unroll
    for (int m = 0; m < 4 * NP; ++m) {
      y0 = __builtin_amdgcn_mfma_f32_16x16x4f32(x.q[m].x, sm[m].x, y0, 0, 0, 0);
      y1 = __builtin_amdgcn_mfma_f32_16x16x4f32(x.q[m].y, sm[m].y, y1, 0, 0, 0);
      y0 = __builtin_amdgcn_mfma_f32_16x16x4f32(x.q[m].z, sm[m].z, y0, 0, 0, 0);
      y1 = __builtin_amdgcn_mfma_f32_16x16x4f32(x.q[m].w, sm[m].w, y1, 0, 0, 0);
      ask_qk(next, src, m);
      __builtin_amdgcn_sched_barrier(0);
    }
#pragma unroll
    for (int T = 0; T < 4; ++T) ask_p(next, src, ahead, T);
#pragma unroll
    for (int T = 0; T < 4; ++T) {
      if (T > w) continue;  // (the same for all lanes)
      y0 = __builtin_amdgcn_mfma_f32_16x16x4f32(x.p[T].x, vm[T].x, y0, 0, 0, 0);
      y1 = __builtin_amdgcn_mfma_f32_16x16x4f32(x.p[T].y, vm[T].y, y1, 0, 0, 0);
      y0 = __builtin_amdgcn_mfma_f32_16x16x4f32(x.p[T].z, vm[T].z, y0, 0, 0, 0);
      y1 = __builtin_amdgcn_mfma_f32_16x16x4f32(x.p[T].w, vm[T].w, y1, 0, 0, 0);
    }
    const int t0 = first + (chunk - c0) * LC_CHUNK + 16 * w + 4 * c;
    float* dst = o + ((size_t)t0 * a.H + h) * a.o_head + j;
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (live && t0 + i < last) dst[(size_t)i * a.H * a.o_head] = y0[i] + y1[i];
    // the state behind the chunk
#pragma unroll
    for (int p = 0; p < NP; ++p) {
      s[p][0] *= x.d[p].x; s[p][1] *= x.d[p].y; s[p][2] *= x.d[p].z; s[p][3] *= x.d[p].w;
    }
#pragma unroll
    for (int T = 0; T < 4; ++T) {
#pragma unroll
      for (int p = 0; p < NP; ++p) s[p] = __builtin_amdgcn_mfma_f32_16x16x4f32(x.k[4 * p + T].x, vm[T].x, s[p], 0, 0, 0);
#pragma unroll
      for (int p = 0; p < NP; ++p) s[p] = __builtin_amdgcn_mfma_f32_16x16x4f32(x.k[4 * p + T].y, vm[T].y, s[p], 0, 0, 0);
#pragma unroll
      for (int p = 0; p < NP; ++p) s[p] = __builtin_amdgcn_mfma_f32_16x16x4f32(x.k[4 * p + T].z, vm[T].z, s[p], 0, 0, 0);
#pragma unroll
      for (int p = 0; p < NP; ++p) s[p] = __builtin_amdgcn_mfma_f32_16x16x4f32(x.k[4 * p + T].w, vm[T].w, s[p], 0, 0, 0);
    }
    __builtin_amdgcn_s_waitcnt(0x0f70);  // vmcnt(0): the next chunk's numbers are there
    hand(next, buf ^ 1);
    __syncthreads();
  };
  LcChunk<NP> xa, xb;
#pragma unroll
  for (int m = 0; m < 4 * NP; ++m) ask_qk(xa, left_by(c0), m);
#pragma unroll
  for (int T = 0; T < 4; ++T) ask_p(xa, left_by(c0), c0, T);
  __builtin_amdgcn_s_waitcnt(0x0f70);
  hand(xa, 0);
  __syncthreads();
#pragma unroll 1
  for (int chunk = c0; chunk < c1; chunk += 2) {
    take(xa, xb, chunk, 0);
    if (chunk + 1 >= c1) break;
    take(xb, xa, chunk + 1, 1);
  }
  if (!live) return;
#pragma unroll
  for (int p = 0; p < NP; ++p)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int n = 16 * (w + 4 * p) + 4 * c + i;
      if (n < a.dk) s_col[n] = s[p][i];
    }
}

// 32-bit words of working memory that a chunk of a step takes for all heads, and a token beside that (the gates).
TK_API int tk_linear_attention_chunk_words(int mode, int H, int dk, int longest) {
  if (!la_chunks_take(mode, dk, longest)) return 0;
  const int dkp = (dk + LC_SLAB - 1) / LC_SLAB * LC_SLAB;
  return (int)(H * lc_words(dkp));
}
TK_API int tk_linear_attention_chunk_tokens() { return LC_CHUNK; }

template <int MODE>
static int lc_run(const LaArgs& a, hipStream_t stream) {
  const int slabs = (a.dk + LC_SLAB - 1) / LC_SLAB, dkp = slabs * LC_SLAB;
  float2* gates = nullptr;
  if (MODE == LA_MEMORY) {
    gates = (float2*)(a.rec + (size_t)a.n_chunks * a.H * lc_words(dkp));
    la_launch_gates(a, gates, 1, stream);
  }
  hipLaunchKernelGGL(la_chunk_factors_kernel<MODE>, dim3(a.n_chunks, a.H), dim3(256), 0, stream, a, dkp, a.proj, gates, a.rec);
  const dim3 grid(a.H, a.n_requests, (la_columns<MODE>(a.dv) + 15) / 16);
#define LC_WALK(NP) hipLaunchKernelGGL((la_chunk_walk_kernel<MODE, NP>), grid, dim3(256), 0, stream, a, a.proj, a.rec, a.o)
  if (slabs == 1) LC_WALK(1);
  else if (slabs == 2) LC_WALK(2);
  else if (slabs == 3) LC_WALK(3);
  else LC_WALK(4);
#undef LC_WALK
  TK_CHECK_LAUNCH("linear_attention");
  return 0;
}

int la_run_chunks(int mode, const LaArgs& a, hipStream_t stream) {
  TK_REQUIRE(a.H < 65536 && a.n_chunks <= a.n_tokens, "linear_attention: bad sizes in chunks");
  return mode == LA_CHANNEL ? lc_run<LA_CHANNEL>(a, stream) : lc_run<LA_MEMORY>(a, stream);
}
