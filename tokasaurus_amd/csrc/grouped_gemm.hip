// Matrix products in which every tile of rows has a weight matrix of its own, on
// v_mfma_f32_16x16x32_bf16: the experts of a mixture (rows sorted by expert) and a matrix a head.
//
//   tk_expert_sort        pairs (token, chosen expert) sorted by expert into slots, every expert's
//                         run of slots filled up to whole tiles of GG_TM or GS_M slots
//   tk_grouped_gemm_bf16  C[c_row(slot), g * c_cols + n] = sum_k W[g][n][k] * A[a_row(slot), g * a_cols + k]
//                         for the slots of every tile, g the tile's group; optionally the gated form
//                         silu(gate) * up of two halves of W[g], or the gated form with clamps
//   tk_expert_sum         per token the weighted sum of its pairs' rows, identity experts, shared expert
//
// A wavefront owns GG_TM = 64 slots x 64 outputs (32 in the gated form, for each of gate and up): weight rows
// are the first operand of the matrix core, read straight from memory 16 bytes a lane, the slots' rows the
// second; a lane ends up with 4 neighbouring outputs of one slot.  The next step's operands are asked for
// before the current step's products.  Where an expert has many rows, tiles of GS_M = 128 slots x 128 weight rows go
// through LDS instead (grouped_gemm_staged_kernel).  Sums are 32-bit and run over k in ascending order for every output:
// a row's result does not depend on which other rows share its tile.
#include <math.h>

#include "common.h"

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8_t;
typedef __attribute__((ext_vector_type(4))) float f32x4_t;

#define GG_TM 64
#define GG_WAVES 4

__device__ __forceinline__ bf16x8_t gg_zero8() {
  bf16x8_t z;
#pragma unroll
  for (int e = 0; e < 8; ++e) z[e] = (__bf16)0.f;
  return z;
}

struct GroupedArgs {
  const bf16_t* A;
  int lda;
  const int* a_row;       // [slots] the row of A a slot reads, < 0: an empty slot; null: the slot's own number
  const int* c_row;       // [slots] the row of C a slot writes, < 0: none; null: the slot's own number
  const int* tile_group;  // [tiles] the group of every tile of slots, < 0: an unused tile, and [tiles] the number of used ones, which come
                          // first; null: blockIdx.z (tiles of GG_TM only)
  int a_cols, c_cols;     // columns of A and C that a group is offset by
  const bf16_t* W;        // [groups][N (2 N in the gated form: gate rows, then up rows)][K]
  size_t w_stride;        // elements from one group's matrix to the next
  void* C;
  int ldc;
  int N, K, slots;
  const float* row_scale;  // (gated form) a factor on a slot's sums of gate and up alike, row_scale[scale_row[slot]]; null: none
  const int* scale_row;
  float limit, alpha;  // (gated form) limit > 0: the activation with clamps (clamped_glu of common.h) instead of silu
};
__device__ __forceinline__ float gg_gated(const GroupedArgs& a, float g, float u) {
  return a.limit > 0.f ? clamped_glu<bf16_t>(g, u, a.limit, a.alpha) : silu_mul_bf16(g, u);
}

// NT: blocks of 16 outputs a wavefront; GLU: the gated form; F32: 32-bit output
template <int NT, bool GLU, bool F32>
__global__ __launch_bounds__(GG_WAVES * TK_WAVE) void grouped_gemm_kernel(GroupedArgs a) {
  constexpr int MB = GG_TM / 16;
  constexpr int WT = GLU ? 2 * NT : NT;  // weight blocks a wavefront reads a step
  const int lane = threadIdx.x & (TK_WAVE - 1), wave = threadIdx.x / TK_WAVE;
  const int tile = blockIdx.x;
  const int g = a.tile_group ? a.tile_group[tile] : (int)blockIdx.z;
  if (g < 0) return;
  const int n0 = (blockIdx.y * GG_WAVES + wave) * NT * 16;
  if (n0 >= a.N) return;
  const int r = lane & 15, q = lane >> 4;
  const bf16_t* Wg = a.W + (size_t)g * a.w_stride;
  const bf16_t* wp[WT];
#pragma unroll
  for (int t = 0; t < WT; ++t) {
    const int blk = GLU ? t % NT : t;
    const int row = min(n0 + blk * 16 + r, a.N - 1) + ((GLU && t >= NT) ? a.N : 0);
    wp[t] = Wg + (size_t)row * a.K + q * 8;
  }
  const bf16_t* ap[MB];
#pragma unroll
  for (int mb = 0; mb < MB; ++mb) {
    const int slot = tile * GG_TM + mb * 16 + r;
    int row = slot < a.slots ? (a.a_row ? a.a_row[slot] : slot) : -1;
    ap[mb] = a.A + (size_t)max(row, 0) * a.lda + (size_t)g * a.a_cols + q * 8;
  }
  f32x4_t acc[WT][MB];
#pragma unroll
  for (int t = 0; t < WT; ++t)
#pragma unroll
    for (int mb = 0; mb < MB; ++mb) acc[t][mb] = f32x4_t{0.f, 0.f, 0.f, 0.f};

  const int steps = (a.K + 31) / 32;
  bf16x8_t w[WT], av[MB];
  auto load = [&](int ks, bf16x8_t (&wv)[WT], bf16x8_t (&xv)[MB]) {
    // a step may reach past K (a multiple of 8): read a valid chunk and zero the weight
    const bool k_ok = ks * 32 + q * 8 < a.K;
    const long off = k_ok ? (long)ks * 32 : -(long)(q * 8);
#pragma unroll
    for (int t = 0; t < WT; ++t) {
      wv[t] = *(const bf16x8_t*)(wp[t] + off);
      if (!k_ok) wv[t] = gg_zero8();
    }
#pragma unroll
    for (int mb = 0; mb < MB; ++mb) xv[mb] = *(const bf16x8_t*)(ap[mb] + off);
  };
  load(0, w, av);
  for (int ks = 0; ks < steps; ++ks) {
    bf16x8_t wn[WT], an[MB];
    if (ks + 1 < steps) load(ks + 1, wn, an);
#pragma unroll
    for (int t = 0; t < WT; ++t)
#pragma unroll
      for (int mb = 0; mb < MB; ++mb)
        acc[t][mb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(w[t], av[mb], acc[t][mb], 0, 0, 0);
    if (ks + 1 < steps) {
#pragma unroll
      for (int t = 0; t < WT; ++t) w[t] = wn[t];
#pragma unroll
      for (int mb = 0; mb < MB; ++mb) av[mb] = an[mb];
    }
  }
  // lane: slot mb * 16 + r, outputs n0 + t * 16 + 4 q + j
#pragma unroll
  for (int mb = 0; mb < MB; ++mb) {
    const int slot = tile * GG_TM + mb * 16 + r;
    if (slot >= a.slots) continue;
    if (a.a_row && a.a_row[slot] < 0) continue;
    const int crow = a.c_row ? a.c_row[slot] : slot;
    if (crow < 0) continue;
    const float f = GLU && a.row_scale ? a.row_scale[a.scale_row[slot]] : 1.f;  // (a slot that is filled names its row)
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      const int n = n0 + t * 16 + 4 * q;
      float y[4];
#pragma unroll
      for (int j = 0; j < 4; ++j) y[j] = GLU ? gg_gated(a, acc[t][mb][j] * f, acc[t + (GLU ? NT : 0)][mb][j] * f) : acc[t][mb][j];
      const size_t at = (size_t)crow * a.ldc + (size_t)g * a.c_cols + n;
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        if (n + j < a.N) {
          if (F32) ((float*)a.C)[at + j] = y[j];
          else ((bf16_t*)a.C)[at + j] = __float2bfloat16(y[j]);
        }
      }
    }
  }
}

// --------------------------------------------------------------------------
// The same product for groups of many slots: a workgroup owns GS_M slots x 128 weight rows (in the gated form 64 of
// gate and the 64 of up that belong to them), its four wavefronts 64 x 64 each.  64 elements of K a step go through LDS in
// two buffers with one barrier a step, 16 bytes a thread and load, the 16-byte pieces of a row exchanged by its number
// (piece ^ (row & 7)) so that the lanes that read one piece of sixteen rows spread over the banks; the next step's
// pieces are on their way to registers meanwhile.  Workgroups go to the chip's dies in turn: each die takes a run of
// neighbouring tiles (an expert's tiles mostly share a die, and its cache the expert's weights), GS_TILES of them at a
// time through all outputs.  Every output's sum runs over k in the order of the kernel above: the same bits.
// --------------------------------------------------------------------------
#define GS_M 128
#define GS_K 64
#define GS_DIES 8
#define GS_TILES 4

__device__ __forceinline__ void gg_store4(bf16_t* dst, const float (&y)[4], int left) {
  union { bf16_t v[4]; uint2 raw; } o;
#pragma unroll
  for (int j = 0; j < 4; ++j) o.v[j] = __float2bfloat16(y[j]);
  if (left >= 4 && ((uintptr_t)dst & 7) == 0) {
    *(uint2*)dst = o.raw;
  } else {
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (j < left) dst[j] = o.v[j];
  }
}

template <bool GLU>
__global__ __launch_bounds__(256, 2) void grouped_gemm_staged_kernel(GroupedArgs a, int tiles, int n_blocks) {
  __shared__ __align__(16) bf16_t sa[2][GS_M * GS_K], sw[2][128 * GS_K];
  const int used = a.tile_group[tiles];  // the tiles that hold slots come first
  const int per = (used + GS_DIES - 1) / GS_DIES;
  const int die = blockIdx.x % GS_DIES, seq = blockIdx.x / GS_DIES;
  const int local = seq / (GS_TILES * n_blocks) * GS_TILES + seq % GS_TILES;
  const int tile = die * per + local;
  if (local >= per || tile >= used) return;
  const int g = a.tile_group[tile];
  if (g < 0) return;
  constexpr int OUT = GLU ? 64 : 128;  // outputs of a workgroup
  const int n0 = seq / GS_TILES % n_blocks * OUT;
  const int lane = threadIdx.x & (TK_WAVE - 1), wave = __builtin_amdgcn_readfirstlane(threadIdx.x / TK_WAVE);
  const int r = lane & 15, q = lane >> 4;
  // what this thread moves: piece `piece` of rows first_row + 32 i
  const int first_row = threadIdx.x / 8, piece = threadIdx.x % 8;
  const bf16_t *ap[4], *wp[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int row = first_row + 32 * i;
    const int slot = tile * GS_M + row;
    const int src = slot < a.slots ? (a.a_row ? a.a_row[slot] : slot) : -1;
    ap[i] = a.A + (size_t)max(src, 0) * a.lda + piece * 8;
    const int wrow = GLU ? min(n0 + (row & 63), a.N - 1) + (row >= 64 ? a.N : 0) : min(n0 + row, a.N - 1);
    wp[i] = a.W + (size_t)g * a.w_stride + (size_t)wrow * a.K + piece * 8;
  }
  const int at = first_row * GS_K + ((piece ^ (first_row & 7)) * 8);  // (the rows 32 apart have the same exchange)
  bf16x8_t pa[4], pw[4];
  auto ask = [&](int k0) {
    // a step may reach past K (a multiple of 8): a valid piece is read and replaced by zeros
    const bool in = k0 + piece * 8 < a.K;
    const long off = in ? (long)k0 : -(long)(piece * 8);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      pa[i] = *(const bf16x8_t*)(ap[i] + off);
      pw[i] = *(const bf16x8_t*)(wp[i] + off);
      if (!in) pw[i] = gg_zero8();
    }
  };
  auto put = [&](int buf) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      *(bf16x8_t*)(sa[buf] + at + 32 * i * GS_K) = pa[i];
      *(bf16x8_t*)(sw[buf] + at + 32 * i * GS_K) = pw[i];
    }
  };
  const int wm = wave & 1, wn = wave >> 1;
  f32x4_t acc[4][4];
#pragma unroll
  for (int t = 0; t < 4; ++t)
#pragma unroll
    for (int mb = 0; mb < 4; ++mb) acc[t][mb] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  auto multiply = [&](int buf) {
#pragma unroll
    for (int kk = 0; kk < 2; ++kk) {
      bf16x8_t w[4], x[4];
      const int swz = ((kk * 4 + q) ^ (r & 7)) * 8;
#pragma unroll
      for (int t = 0; t < 4; ++t) {
        // gated: blocks 0, 1 of gate and 2, 3 of up
        const int row = GLU ? (t >> 1) * 64 + wn * 32 + (t & 1) * 16 + r : wn * 64 + t * 16 + r;
        w[t] = *(const bf16x8_t*)(sw[buf] + row * GS_K + swz);
      }
#pragma unroll
      for (int mb = 0; mb < 4; ++mb) x[mb] = *(const bf16x8_t*)(sa[buf] + (wm * 64 + mb * 16 + r) * GS_K + swz);
#pragma unroll
      for (int t = 0; t < 4; ++t)
#pragma unroll
        for (int mb = 0; mb < 4; ++mb) acc[t][mb] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(w[t], x[mb], acc[t][mb], 0, 0, 0);
    }
  };
  ask(0);
  put(0);
  __syncthreads();
  int buf = 0;
  for (int k0 = 0; k0 < a.K; k0 += GS_K, buf ^= 1) {
    const bool more = k0 + GS_K < a.K;
    if (more) ask(k0 + GS_K);
    multiply(buf);
    if (more) put(buf ^ 1);
    __syncthreads();
  }
  // lane: slot wm * 64 + mb * 16 + r, outputs 4 q + j of a block
#pragma unroll
  for (int mb = 0; mb < 4; ++mb) {
    const int slot = tile * GS_M + wm * 64 + mb * 16 + r;
    if (slot >= a.slots) continue;
    if (a.a_row && a.a_row[slot] < 0) continue;
    const int crow = a.c_row ? a.c_row[slot] : slot;
    if (crow < 0) continue;
    const float f = GLU && a.row_scale ? a.row_scale[a.scale_row[slot]] : 1.f;
    bf16_t* dst = (bf16_t*)a.C + (size_t)crow * a.ldc;
#pragma unroll
    for (int t = 0; t < (GLU ? 2 : 4); ++t) {
      const int n = n0 + (GLU ? wn * 32 + t * 16 : wn * 64 + t * 16) + 4 * q;
      float y[4];
#pragma unroll
      for (int j = 0; j < 4; ++j) y[j] = GLU ? gg_gated(a, acc[t][mb][j] * f, acc[t + (GLU ? 2 : 0)][mb][j] * f) : acc[t][mb][j];
      if (n < a.N) gg_store4(dst + n, y, a.N - n);
    }
  }
}

TK_API int tk_grouped_gemm_bf16(const void* A, int lda, const int* a_row, const int* c_row, const int* tile_group, int tiles,
                                int groups_z, int a_cols, int c_cols, const void* W, size_t w_stride, void* C, int ldc,
                                int N, int K, int slots, int glu, int out_f32, const float* row_scale, const int* scale_row,
                                int tile_slots, float limit, float alpha, hipStream_t stream) {
  TK_REQUIRE(A && W && C && N > 0 && K > 0 && slots >= 0 && tiles >= 0, "grouped_gemm: bad arguments");
  TK_REQUIRE(K % 8 == 0 && lda % 8 == 0 && a_cols % 8 == 0 && w_stride % 8 == 0 && (((uintptr_t)A | (uintptr_t)W) & 15) == 0,
             "grouped_gemm: rows of A and W must start at multiples of 16 bytes (K=%d lda=%d)", K, lda);
  TK_REQUIRE((tile_group != nullptr) != (groups_z > 0), "grouped_gemm: groups come by tile or by the grid, not both");
  TK_REQUIRE(!row_scale || (glu && scale_row && a_row), "grouped_gemm: a factor a row goes with the gated form and rows by slot");
  TK_REQUIRE(!(glu && out_f32), "grouped_gemm: the gated form writes the storage type");
  if (tiles == 0 || slots == 0) return 0;
  GroupedArgs a{(const bf16_t*)A, lda, a_row, c_row, tile_group, a_cols, c_cols, (const bf16_t*)W, w_stride, C, ldc, N, K, slots,
                row_scale, scale_row, limit, alpha};
  TK_REQUIRE(tile_slots == GG_TM || (tile_slots == GS_M && tile_group && !out_f32 && a_cols == 0 && c_cols == 0),
             "grouped_gemm: tiles of %d slots, or of %d with groups by tile and storage-type output", GG_TM, GS_M);
  if (tile_slots == GS_M) {
    const int outs = glu ? 64 : 128;
    const int n_blocks = (N + outs - 1) / outs, per = (tiles + GS_DIES - 1) / GS_DIES;
    const long groups = (long)GS_DIES * ((per + GS_TILES - 1) / GS_TILES) * GS_TILES * n_blocks;
    TK_REQUIRE(groups < (1l << 31), "grouped_gemm: too many outputs");
    if (glu) hipLaunchKernelGGL(grouped_gemm_staged_kernel<true>, dim3((unsigned)groups), dim3(256), 0, stream, a, tiles, n_blocks);
    else hipLaunchKernelGGL(grouped_gemm_staged_kernel<false>, dim3((unsigned)groups), dim3(256), 0, stream, a, tiles, n_blocks);
    TK_CHECK_LAUNCH("grouped_gemm");
    return 0;
  }
  const int nt = glu ? 2 : 4;
  const dim3 grid(tiles, (N + GG_WAVES * nt * 16 - 1) / (GG_WAVES * nt * 16), groups_z > 0 ? groups_z : 1);
  TK_REQUIRE(grid.y < 65536 && grid.z < 65536, "grouped_gemm: too many outputs or groups");
  if (glu)
    hipLaunchKernelGGL((grouped_gemm_kernel<2, true, false>), grid, dim3(GG_WAVES * TK_WAVE), 0, stream, a);
  else if (out_f32)
    hipLaunchKernelGGL((grouped_gemm_kernel<4, false, true>), grid, dim3(GG_WAVES * TK_WAVE), 0, stream, a);
  else
    hipLaunchKernelGGL((grouped_gemm_kernel<4, false, false>), grid, dim3(GG_WAVES * TK_WAVE), 0, stream, a);
  TK_CHECK_LAUNCH("grouped_gemm");
  return 0;
}

// --------------------------------------------------------------------------
// Pairs (token, place) -> slots sorted by expert.  A workgroup a job: a layer's choice, or (where the choice of several layers
// is known before the first of them runs) all layers' in one launch.  Expert e's pairs take the slots
// first[e] .. first[e] + count[e] - 1 with first[e] a multiple of tm; the slots between a run's end and the
// next multiple are empty.  slot_pair[slot] = the pair (or -1), slot_token[slot] = its token (or -1),
// tile_group[tile] = the expert whose run the tile lies in (or -1), tile_group[max_tiles] = the tiles in use.  Pairs of identity experts (ids >= experts)
// and empty places (ids < 0) get no slot.  Which of an expert's slots a pair gets depends on the order of
// arrival and changes no result: every row is computed on its own.
// --------------------------------------------------------------------------
struct SortJob {
  const int* ids;
  int *slot_pair, *slot_token, *tile_group;
  int pairs, top, experts, max_tiles, tm;
};
#define SORT_JOBS 48
struct SortJobs {
  SortJob job[SORT_JOBS];
};
__global__ __launch_bounds__(1024) void expert_sort_kernel(SortJobs jobs) {
  const SortJob& jb = jobs.job[blockIdx.x];
  const int* __restrict__ ids = jb.ids;
  const int pairs = jb.pairs, top = jb.top, experts = jb.experts, max_tiles = jb.max_tiles, tm = jb.tm;
  int* __restrict__ slot_pair = jb.slot_pair;
  int* __restrict__ slot_token = jb.slot_token;
  int* __restrict__ tile_group = jb.tile_group;
  extern __shared__ int sh[];  // [experts] counts, [experts] first slots, [experts] cursors
  int* count = sh;
  int* first = sh + experts;
  int* cursor = sh + 2 * experts;
  for (int e = threadIdx.x; e < experts; e += blockDim.x) count[e] = cursor[e] = 0;
  for (int s = threadIdx.x; s < max_tiles * tm; s += blockDim.x) slot_pair[s] = slot_token[s] = -1;
  for (int t = threadIdx.x; t < max_tiles; t += blockDim.x) tile_group[t] = -1;
  __syncthreads();
  for (int p = threadIdx.x; p < pairs; p += blockDim.x) {
    const int e = ids[p];
    if (e >= 0 && e < experts) atomicAdd(&count[e], 1);
  }
  __syncthreads();
  if (threadIdx.x == 0) {
    int at = 0;
    for (int e = 0; e < experts; ++e) {
      first[e] = at;
      at += (count[e] + tm - 1) / tm * tm;
    }
    tile_group[max_tiles] = at / tm;
  }
  __syncthreads();
  for (int e = threadIdx.x; e < experts; e += blockDim.x)
    for (int t = first[e] / tm; t < (first[e] + count[e] + tm - 1) / tm; ++t) tile_group[t] = e;
  for (int p = threadIdx.x; p < pairs; p += blockDim.x) {
    const int e = ids[p];
    if (e >= 0 && e < experts) {
      const int s = first[e] + atomicAdd(&cursor[e], 1);
      slot_pair[s] = p;
      slot_token[s] = p / top;
    }
  }
}

TK_API int tk_expert_sort(const SortJob* jobs, int n_jobs, hipStream_t stream) {
  TK_REQUIRE(jobs && n_jobs >= 0, "expert_sort: bad arguments");
  for (int first = 0; first < n_jobs; first += SORT_JOBS) {
    SortJobs all{};
    const int n = min(SORT_JOBS, n_jobs - first);
    int most = 0;
    for (int k = 0; k < n; ++k) {
      const SortJob& j = all.job[k] = jobs[first + k];
      TK_REQUIRE(j.ids && j.slot_pair && j.slot_token && j.tile_group && j.pairs >= 0 && j.top > 0 && j.experts > 0, "expert_sort: bad arguments");
      TK_REQUIRE(j.tm == GG_TM || j.tm == GS_M, "expert_sort: tiles of %d slots", j.tm);
      TK_REQUIRE(j.max_tiles >= (j.pairs + j.tm - 1) / j.tm + j.experts, "expert_sort: %d tiles cannot hold %d pairs of %d experts", j.max_tiles,
                 j.pairs, j.experts);
      TK_REQUIRE(3 * j.experts * sizeof(int) <= 48 * 1024, "expert_sort: too many experts");
      most = max(most, j.experts);
    }
    hipLaunchKernelGGL(expert_sort_kernel, dim3(n), dim3(1024), 3 * most * sizeof(int), stream, all);
    TK_CHECK_LAUNCH("expert_sort");
  }
  return 0;
}

// --------------------------------------------------------------------------
// out[t, c] = sum over the places k of token t, in order, of weights[t, k] * (y[t * top + k, c] for a routed expert,
// h[t, c] for an identity expert), plus shared_gate[t] * shared[t, c].  y: [pairs, width] in the storage type.
// `unit` != 0: a routed expert's row is added as it is.  weights null: equal parts, 1 / top each.
// --------------------------------------------------------------------------
__global__ __launch_bounds__(256) void expert_sum_kernel(const bf16_t* __restrict__ h, int h_stride, const bf16_t* __restrict__ y,
                                                         const int* __restrict__ ids, const float* __restrict__ weights,
                                                         const float* __restrict__ shared, const float* __restrict__ shared_gate,
                                                         float* __restrict__ out, int width, int experts, int top, int unit) {
  const int t = blockIdx.x;
  for (int c = threadIdx.x; c < width; c += blockDim.x) {
    float acc = 0.f;
    for (int k = 0; k < top; ++k) {
      const int e = ids[(size_t)t * top + k];
      if (e < 0) continue;
      const float v = e < experts ? __bfloat162float(y[((size_t)t * top + k) * width + c]) : __bfloat162float(h[(size_t)t * h_stride + c]);
      acc = fmaf(unit && e < experts ? 1.f : (weights ? weights[(size_t)t * top + k] : 1.0f / (float)top), v, acc);
    }
    if (shared) acc = fmaf(shared_gate[t], shared[(size_t)t * width + c], acc);
    out[(size_t)t * width + c] = acc;
  }
}

// The same with 16 bytes a load, a thread eight neighbouring columns, and all of a token's rows asked for before the first is
// used (EXPERT_SUM_TOP at a time).
#define EXPERT_SUM_TOP 4
__global__ __launch_bounds__(256) void expert_sum_vec_kernel(const bf16_t* __restrict__ h, int h_stride, const bf16_t* __restrict__ y,
                                                             const int* __restrict__ ids, const float* __restrict__ weights,
                                                             const float* __restrict__ shared, const float* __restrict__ shared_gate,
                                                             float* __restrict__ out, int width, int experts, int top, int unit) {
  const size_t t = blockIdx.x;
  for (int c = threadIdx.x * 8; c < width; c += blockDim.x * 8) {
    float acc[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) acc[j] = 0.f;
    for (int k0 = 0; k0 < top; k0 += EXPERT_SUM_TOP) {
      uint4 raw[EXPERT_SUM_TOP];
      float f[EXPERT_SUM_TOP];
#pragma unroll
      for (int k = 0; k < EXPERT_SUM_TOP; ++k) {
        f[k] = 0.f;
        raw[k] = make_uint4(0, 0, 0, 0);
        if (k0 + k >= top) continue;
        const int e = ids[t * top + k0 + k];
        if (e < 0) continue;
        f[k] = unit && e < experts ? 1.f : (weights ? weights[t * top + k0 + k] : 1.0f / (float)top);
        raw[k] = e < experts ? *(const uint4*)(y + (t * top + k0 + k) * width + c) : *(const uint4*)(h + t * h_stride + c);
      }
#pragma unroll
      for (int k = 0; k < EXPERT_SUM_TOP; ++k) {
        const bf16_t* v = (const bf16_t*)&raw[k];
#pragma unroll
        for (int j = 0; j < 8; ++j) acc[j] = fmaf(f[k], __bfloat162float(v[j]), acc[j]);
      }
    }
    if (shared) {
      const float s = shared_gate[t];
#pragma unroll
      for (int j = 0; j < 8; ++j) acc[j] = fmaf(s, shared[t * width + c + j], acc[j]);
    }
    *(float4*)(out + t * width + c) = make_float4(acc[0], acc[1], acc[2], acc[3]);
    *(float4*)(out + t * width + c + 4) = make_float4(acc[4], acc[5], acc[6], acc[7]);
  }
}

TK_API int tk_expert_sum(const void* h, int h_stride, const void* y, const int* ids, const float* weights, const float* shared,
                         const float* shared_gate, float* out, int tokens, int width, int experts, int top, int unit, hipStream_t stream) {
  TK_REQUIRE(h && y && ids && out && (!shared || shared_gate) && tokens >= 0 && width > 0 && top > 0 && h_stride >= width,
             "expert_sum: bad arguments");
  if (tokens == 0) return 0;
  if (width % 8 == 0 && h_stride % 8 == 0 && (((uintptr_t)h | (uintptr_t)y | (uintptr_t)out | (uintptr_t)shared) & 15) == 0) {
    hipLaunchKernelGGL(expert_sum_vec_kernel, dim3(tokens), dim3(256), 0, stream, (const bf16_t*)h, h_stride, (const bf16_t*)y, ids,
                       weights, shared, shared_gate, out, width, experts, top, unit);
    TK_CHECK_LAUNCH("expert_sum");
    return 0;
  }
  hipLaunchKernelGGL(expert_sum_kernel, dim3(tokens), dim3(256), 0, stream, (const bf16_t*)h, h_stride, (const bf16_t*)y, ids,
                     weights, shared, shared_gate, out, width, experts, top, unit);
  TK_CHECK_LAUNCH("expert_sum");
  return 0;
}
