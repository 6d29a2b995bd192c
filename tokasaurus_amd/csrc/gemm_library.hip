// Library matrix products (hipBLASLt) for more rows than the weight-streaming kernel takes:
// out[M, N] = x[M, K] . w[N, K]^T in bfloat16 with 32-bit accumulation, the result in bfloat16
// or in 32-bit.  The library is asked once per problem (sizes, leading dimensions, output type)
// which of its kernels it thinks fastest; the answer and the problem's descriptors are kept, so
// that a later call of the same problem costs one hipblasLtMatmul and nothing else on the host
// (10 us against the 18 us of a product through the tensor library's dispatcher: a prompt
// portion of a few hundred tokens is bound by the host's launches, 61 of which are products).
// The kernel chosen is the one the tensor library's own product gets from the same question.
//
// No device memory is allocated here: the caller brings the workspace that the library's
// kernels may use (stream-K partial sums), the same for every call on a stream.  A device's calls are to be on one stream at
// a time: they share a handle, and a stream-K kernel's workgroups wait for one another.
#include "common.h"

#include <hipblaslt/hipblaslt.h>

#include <map>
#include <mutex>
#include <tuple>

namespace {

struct Problem {
  hipblasLtMatmulDesc_t desc = nullptr;
  hipblasLtMatrixLayout_t w = nullptr, x = nullptr, out = nullptr;
  hipblasLtMatmulAlgo_t algo;
  size_t workspace = 0;
};

using Key = std::tuple<int, int, int, int, int, int, int, int, size_t>;  // device, M, N, K, ldx, ldw, ldo, f32, workspace

std::mutex g_lock;
std::map<int, hipblasLtHandle_t> g_handles;  // one a device
std::map<Key, Problem> g_problems;
constexpr size_t MAX_PROBLEMS = 8192;  // beyond that all are forgotten and asked for again

void destroy(Problem& p) {
  if (p.w) hipblasLtMatrixLayoutDestroy(p.w);
  if (p.x) hipblasLtMatrixLayoutDestroy(p.x);
  if (p.out) hipblasLtMatrixLayoutDestroy(p.out);
  if (p.desc) hipblasLtMatmulDescDestroy(p.desc);
  p = Problem();
}

// In the library's column-major terms: out^T [N, M] = w^T (w stored [K, N], transposed) . x^T
// (stored [K, M]).  Returns 0, or the step that failed.
int describe(hipblasLtHandle_t handle, Problem& p, int M, int N, int K, int ldx, int ldw, int ldo, int f32, size_t workspace) {
  if (hipblasLtMatmulDescCreate(&p.desc, HIPBLAS_COMPUTE_32F, HIP_R_32F) != HIPBLAS_STATUS_SUCCESS) return 1;
  const int32_t transposed = HIPBLAS_OP_T, plain = HIPBLAS_OP_N;
  if (hipblasLtMatmulDescSetAttribute(p.desc, HIPBLASLT_MATMUL_DESC_TRANSA, &transposed, sizeof transposed) != HIPBLAS_STATUS_SUCCESS) return 2;
  if (hipblasLtMatmulDescSetAttribute(p.desc, HIPBLASLT_MATMUL_DESC_TRANSB, &plain, sizeof plain) != HIPBLAS_STATUS_SUCCESS) return 2;
  if (hipblasLtMatrixLayoutCreate(&p.w, HIP_R_16BF, K, N, ldw) != HIPBLAS_STATUS_SUCCESS) return 3;
  if (hipblasLtMatrixLayoutCreate(&p.x, HIP_R_16BF, K, M, ldx) != HIPBLAS_STATUS_SUCCESS) return 3;
  if (hipblasLtMatrixLayoutCreate(&p.out, f32 ? HIP_R_32F : HIP_R_16BF, N, M, ldo) != HIPBLAS_STATUS_SUCCESS) return 3;
  hipblasLtMatmulPreference_t pref = nullptr;
  if (hipblasLtMatmulPreferenceCreate(&pref) != HIPBLAS_STATUS_SUCCESS) return 4;
  const uint64_t room = workspace;
  hipblasLtMatmulPreferenceSetAttribute(pref, HIPBLASLT_MATMUL_PREF_MAX_WORKSPACE_BYTES, &room, sizeof room);
  // the library's candidates, fastest first by its own estimate; the first whose workspace fits
  // is taken (a stream-K kernel's partial sums want up to 64 MB, whatever room was named)
  constexpr int ASKED = 8;
  hipblasLtMatmulHeuristicResult_t found[ASKED];
  int n = 0;
  const hipblasStatus_t st = hipblasLtMatmulAlgoGetHeuristic(handle, p.desc, p.w, p.x, p.out, p.out, pref, ASKED, found, &n);
  hipblasLtMatmulPreferenceDestroy(pref);
  if (st != HIPBLAS_STATUS_SUCCESS || n < 1) return 5;
  for (int i = 0; i < n; ++i) {
    if (found[i].state == HIPBLAS_STATUS_SUCCESS && found[i].workspaceSize <= workspace) {
      p.algo = found[i].algo;
      p.workspace = found[i].workspaceSize;
      return 0;
    }
  }
  return 6;
}

}  // namespace

// out [M, N] (rows ldo apart; bfloat16, or 32-bit when f32_out) = x [M, K] (rows ldx apart) .
// w [N, K]^T (rows ldw apart), both bfloat16.  workspace: device memory of workspace_bytes
// (16-byte aligned) that the library's kernel may use; calls on one stream may share it.
TK_API int tk_gemm_library_bf16(const void* x, int ldx, const void* w, int ldw, void* out, int ldo, int M, int N, int K,
                                int f32_out, void* workspace, size_t workspace_bytes, hipStream_t stream) {
  TK_REQUIRE(M > 0 && N > 0 && K > 0 && ldx >= K && ldw >= K && ldo >= N, "gemm_library: bad sizes M=%d N=%d K=%d ldx=%d ldw=%d ldo=%d",
             M, N, K, ldx, ldw, ldo);
  TK_REQUIRE(x && w && out, "gemm_library: null operand");
  TK_REQUIRE(workspace_bytes == 0 || (workspace && ((uintptr_t)workspace & 15) == 0), "gemm_library: the workspace must be 16-byte aligned");
  int device = 0;
  TK_REQUIRE(hipGetDevice(&device) == hipSuccess, "gemm_library: no current device");
  std::lock_guard<std::mutex> guard(g_lock);
  auto h = g_handles.find(device);
  if (h == g_handles.end()) {
    hipblasLtHandle_t handle = nullptr;
    TK_REQUIRE(hipblasLtCreate(&handle) == HIPBLAS_STATUS_SUCCESS, "gemm_library: hipblasLtCreate failed");
    h = g_handles.emplace(device, handle).first;
  }
  const Key key(device, M, N, K, ldx, ldw, ldo, f32_out != 0, workspace_bytes);
  auto it = g_problems.find(key);
  if (it == g_problems.end()) {
    if (g_problems.size() >= MAX_PROBLEMS) {
      for (auto& kv : g_problems) destroy(kv.second);
      g_problems.clear();
    }
    Problem p;
    const int step = describe(h->second, p, M, N, K, ldx, ldw, ldo, f32_out != 0, workspace_bytes);
    if (step != 0) {
      destroy(p);
      TK_REQUIRE(false, "gemm_library: the library has no kernel for M=%d N=%d K=%d (ldx=%d ldw=%d ldo=%d, %s output, %zu bytes of workspace; step %d)",
                 M, N, K, ldx, ldw, ldo, f32_out ? "32-bit" : "bfloat16", workspace_bytes, step);
    }
    it = g_problems.emplace(key, p).first;
  }
  const Problem& p = it->second;
  const float one = 1.0f, zero = 0.0f;
  const hipblasStatus_t st = hipblasLtMatmul(h->second, p.desc, &one, w, p.w, x, p.x, &zero, out, p.out, out, p.out, &p.algo, workspace,
                                             workspace_bytes, stream);
  TK_REQUIRE(st == HIPBLAS_STATUS_SUCCESS, "gemm_library: hipblasLtMatmul failed with status %d (M=%d N=%d K=%d)", (int)st, M, N, K);
  return 0;
}
