// Instantiations of the prefill GEMMs (gemm_impl.h) for bf16 (N, K) weights, and the plain products of
// models whose residual is not bf16: activation epilogues and a split-K form without a residual.
#include "gemm_impl.h"

namespace llj {

template <int EP>
static int bf16_run(const GemmParams& p, hipStream_t s) {
  if (p.M >= 256 && glds_enabled(GWF_BF16)) return gemm_glds_run<GWF_BF16, EP>(p, s);
  if (LLJ_GEMM_BM256 && p.M >= 256) return gemm_launch<GWF_BF16, EP, 256>(p, s);
  return gemm_launch<GWF_BF16, EP>(p, s);
}

int gemm_bf16_run(int ep, const GemmParams& p, hipStream_t s) {
  switch (ep) {
    case GEP_STORE: return bf16_run<GEP_STORE>(p, s);
    case GEP_RESID: return bf16_run<GEP_RESID>(p, s);
    case GEP_QKV: return bf16_run<GEP_QKV>(p, s);
    case GEP_SILU_MUL: return bf16_run<GEP_SILU_MUL>(p, s);
    case GEP_RELU2: return bf16_run<GEP_RELU2>(p, s);
    case GEP_BIAS: return bf16_run<GEP_BIAS>(p, s);
    case GEP_GLU: return bf16_run<GEP_GLU>(p, s);
    case GEP_PARTIAL: return gemm_glds_launch<GWF_BF16, GEP_PARTIAL, 128>(p, s);
  }
  return LLJ_EINVAL;
}

// C = bf16(sum over the slices of their fp32 partials + bias), slices in order
__global__ __launch_bounds__(256) void gemm_splitk_store_kernel(const float* __restrict__ ws, int nsplit, int M, int N,
                                                                const float* __restrict__ bias, bf16_t* __restrict__ C, int ldc) {
  const size_t i = ((size_t)blockIdx.x * 256 + threadIdx.x) * 4;
  if (i >= (size_t)M * N) return;
  const int m = (int)(i / N), n = (int)(i % N);
  float4 y = *reinterpret_cast<const float4*>(ws + i);
  for (int sp = 1; sp < nsplit; ++sp) {
    const float4 v = *reinterpret_cast<const float4*>(ws + (size_t)sp * M * N + i);
    y.x += v.x; y.y += v.y; y.z += v.z; y.w += v.w;
  }
  if (bias) {
    const float4 b = *reinterpret_cast<const float4*>(bias + n);
    y.x += b.x; y.y += b.y; y.z += b.z; y.w += b.w;
  }
  *reinterpret_cast<uint2*>(C + (size_t)m * ldc + n) = make_uint2(pack2bf(y.x, y.y), pack2bf(y.z, y.w));
}

}  // namespace llj

using namespace llj;

extern "C" {
LLJ_TRACE_EXPORT(gemm_bf16)

size_t llj_gemm_bf16_ws_bytes(int M, int N, int K) {
  int kcs = 0;
  const int ns = splitk_plan(GWF_BF16, M, N, K, &kcs);
  return ns ? (size_t)ns * M * N * sizeof(float) : 0;
}

int llj_gemm_bf16(int act, const void* A, int lda, const void* W, const float* bias, void* C, int ldc, int M, int N, int K,
                  float limit, float alpha, void* ws, size_t ws_bytes, void* stream) {
  LLJ_REQUIRE(act >= 0 && act <= 2 && (act != 1 || !bias) && A && W && C && M > 0 && N % kGBN == 0 && K % 128 == 0 && N > 0 &&
              K > 0 && lda >= K && ldc >= (act == 2 ? N / 2 : N) && (lda & 7) == 0 && (ldc & 3) == 0 &&
              ((uintptr_t)bias & 15) == 0);
  GemmParams p{};
  p.A = (const bf16_t*)A; p.lda = lda; p.M = M; p.N = N; p.K = K; p.W = W; p.C = (bf16_t*)C; p.ldc = ldc;
  p.bias = bias; p.limit = limit; p.alpha = alpha;
  hipStream_t s = (hipStream_t)stream;
  int kcs = 0;
  const int ns = act == 0 && ws ? splitk_plan(GWF_BF16, M, N, K, &kcs) : 0;
  if (!ns) return gemm_bf16_run(act == 2 ? GEP_GLU : act ? GEP_RELU2 : bias ? GEP_BIAS : GEP_STORE, p, s);
  LLJ_REQUIRE(ws_bytes >= (size_t)ns * M * N * sizeof(float));
  p.ws = (float*)ws; p.nsplit = ns; p.kcs = kcs;
  if (const int rc = gemm_bf16_run(GEP_PARTIAL, p, s)) return rc;
  const size_t n4 = (size_t)M * N / 4;
  hipLaunchKernelGGL(gemm_splitk_store_kernel, dim3((unsigned)((n4 + 255) / 256)), dim3(256), 0, s, (const float*)ws, ns, M,
                     N, bias, (bf16_t*)C, ldc);
  LLJ_CHECK_LAUNCH();
  return 0;
}

}  // extern "C"
