// Residual-side ops of models whose residual is several streams (hyper-connections): a sublayer reads
// u = sum_s in[s] x_s through a layer norm, and leaves x'_t = sum_s mix[s][t] x_s + out[t] y, every stream from the
// old ones. The end of one sublayer and the start of the next are one pass over the streams: they are read
// and written once per sublayer. Streams, norms and sums are fp32; y, the norm weight and the normed rows h have the
// activation type (dt 0 bf16, 1 fp32). x is [rows][streams][ldx]; columns of h past the width are written as zeros.
#include "common.h"
#include "elem.h"
#include "lit_llama_amd.h"

namespace llj {

struct StreamsParams {
  // the start of the streams: embed[tok] * scale in all of them (tok != NULL), or the end of a sublayer
  const int* tok;
  const void* embed;
  int lde;
  float scale;
  int* pos;  // decode rows: advanced by one (with tok)
  const void* y;
  int ldy;
  const float* out;  // [S]
  const float* mix;  // [S][S], from, to
  float* x;
  int ldx;
  const float* in;  // [S]; NULL: the plain sum
  const void* w;
  float eps;
  void* h;
  int ldh;
  const int* rows;  // output row i is of row rows[i], and x stays as it is
  int S, C;
};

constexpr int kFewRows = 64;

template <int NW>
__device__ __forceinline__ float block_sum(float v, float* red) {
  v = wave_sum(v);
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  float s = 0.f;
#pragma unroll
  for (int i = 0; i < NW; ++i) s += red[i];
  __syncthreads();
  return s;
}

// VW (8 or 4) consecutive elements
template <int VW, typename T>
__device__ __forceinline__ void ldw(const T* p, float (&o)[VW]) {
  if constexpr (VW == 8) {
    ld8(p, o);
  } else if constexpr (sizeof(T) == 2) {
    const uint2 v = *reinterpret_cast<const uint2*>(p);
    o[0] = bflo(v.x); o[1] = bfhi(v.x); o[2] = bflo(v.y); o[3] = bfhi(v.y);
  } else {
    const float4 v = *reinterpret_cast<const float4*>(p);
    o[0] = v.x; o[1] = v.y; o[2] = v.z; o[3] = v.w;
  }
}
template <int VW, typename T>
__device__ __forceinline__ void stw(T* p, const float (&v)[VW]) {
  if constexpr (VW == 8) st8(p, v);
  else if constexpr (sizeof(T) == 2) *reinterpret_cast<uint2*>(p) = make_uint2(pack2bf(v[0], v[1]), pack2bf(v[2], v[3]));
  else *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
}

// One workgroup of NT threads per row, VW columns per thread and step, widths up to VW * NT * NV held in registers. Many
// rows: 256 threads of 8 columns; few rows (decode steps): 1024 of 4, a row's loads spread over more waves.
template <typename T, int S, int NV, int NT, int VW>
__global__ __launch_bounds__(NT) void streams_kernel(StreamsParams p) {
  constexpr int NW = NT / 64;
  __shared__ float red[NW];
  const int i = blockIdx.x, tid = threadIdx.x, C = p.C;
  const size_t m = p.rows ? p.rows[i] : i;
  float* xr = p.x + m * S * p.ldx;
  const T* yr = p.tok ? (const T*)p.embed + (size_t)p.tok[m] * p.lde : (const T*)p.y + m * p.ldy;
  if (p.tok && p.pos && tid == 0) p.pos[i] += 1;
  float u[NV][VW], wv[NV][VW];
  float sum = 0.f;
#pragma unroll
  for (int v = 0; v < NV; ++v) {
    const int k = VW * (tid + NT * v);
#pragma unroll
    for (int e = 0; e < VW; ++e) u[v][e] = 0.f;
    if (k < C) {
      float y[VW], x[S][VW];
      ldw<VW>(yr + k, y);
      ldw<VW>((const T*)p.w + k, wv[v]);
      if (!p.tok) {
#pragma unroll
        for (int s = 0; s < S; ++s) ldw<VW>(xr + (size_t)s * p.ldx + k, x[s]);
      }
#pragma unroll
      for (int t = 0; t < S; ++t) {
        const float in = p.in ? p.in[t] : 1.f;
        float n[VW];
        if (p.tok) {
#pragma unroll
          for (int e = 0; e < VW; ++e) n[e] = y[e] * p.scale;
        } else {
          const float ot = p.out[t];
#pragma unroll
          for (int e = 0; e < VW; ++e) n[e] = ot * y[e];
#pragma unroll
          for (int s = 0; s < S; ++s) {
            const float a = p.mix[s * S + t];
#pragma unroll
            for (int e = 0; e < VW; ++e) n[e] += a * x[s][e];
          }
        }
        if (!p.rows) stw<VW>(xr + (size_t)t * p.ldx + k, n);
#pragma unroll
        for (int e = 0; e < VW; ++e) u[v][e] += in * n[e];
      }
#pragma unroll
      for (int e = 0; e < VW; ++e) sum += u[v][e];
    }
  }
  const float mean = block_sum<NW>(sum, red) / (float)C;
  sum = 0.f;
#pragma unroll
  for (int v = 0; v < NV; ++v)
    if (VW * (tid + NT * v) < C) {
#pragma unroll
      for (int e = 0; e < VW; ++e) {
        u[v][e] -= mean;
        sum += u[v][e] * u[v][e];
      }
    }
  const float rs = 1.f / sqrtf(block_sum<NW>(sum, red) / (float)C + p.eps);
  T* hr = (T*)p.h + (size_t)i * p.ldh;
#pragma unroll
  for (int v = 0; v < NV; ++v) {
    const int k = VW * (tid + NT * v);
    if (k < C) {
#pragma unroll
      for (int e = 0; e < VW; ++e) u[v][e] *= rs * wv[v][e];
      stw<VW>(hr + k, u[v]);
    }
  }
  for (int k = C + tid; k < p.ldh; k += NT) stv(hr, k, 0.f);
}

// Any width and number of streams: a column at a time, its old streams in the thread's own LDS words (so the
// update is in place), the mixed row u in LDS.
template <typename T>
__global__ __launch_bounds__(256) void streams_any_kernel(StreamsParams p) {
  extern __shared__ __attribute__((aligned(16))) float smem_f[];
  __shared__ float red[4];
  float* u = smem_f;         // [C]
  float* old = u + p.C;      // [S][256]
  const int i = blockIdx.x, tid = threadIdx.x, C = p.C, S = p.S;
  const size_t m = p.rows ? p.rows[i] : i;
  float* xr = p.x + m * S * p.ldx;
  const T* yr = p.tok ? (const T*)p.embed + (size_t)p.tok[m] * p.lde : (const T*)p.y + m * p.ldy;
  if (p.tok && p.pos && tid == 0) p.pos[i] += 1;
  float sum = 0.f;
  for (int k = tid; k < C; k += 256) {
    const float y = ldv(yr, k);
    if (!p.tok)
      for (int s = 0; s < S; ++s) old[s * 256 + tid] = xr[(size_t)s * p.ldx + k];
    float a = 0.f;
    for (int t = 0; t < S; ++t) {
      float n = p.tok ? y * p.scale : p.out[t] * y;
      if (!p.tok)
        for (int s = 0; s < S; ++s) n += p.mix[s * S + t] * old[s * 256 + tid];
      if (!p.rows) xr[(size_t)t * p.ldx + k] = n;
      a += (p.in ? p.in[t] : 1.f) * n;
    }
    u[k] = a;
    sum += a;
  }
  const float mean = block_sum<4>(sum, red) / (float)C;
  sum = 0.f;
  for (int k = tid; k < C; k += 256) sum += (u[k] - mean) * (u[k] - mean);
  const float rs = 1.f / sqrtf(block_sum<4>(sum, red) / (float)C + p.eps);
  T* hr = (T*)p.h + (size_t)i * p.ldh;
  for (int k = tid; k < p.ldh; k += 256) stv(hr, k, k < C ? (u[k] - mean) * rs * ldv((const T*)p.w, k) : 0.f);
}

template <typename T, int S>
static int streams_wide(const StreamsParams& p, int M, hipStream_t s) {
  if (M <= kFewRows && p.C <= 4096) hipLaunchKernelGGL((streams_kernel<T, S, 1, 1024, 4>), dim3(M), dim3(1024), 0, s, p);
  else if (p.C <= 2048) hipLaunchKernelGGL((streams_kernel<T, S, 1, 256, 8>), dim3(M), dim3(256), 0, s, p);
  else if (p.C <= 4096) hipLaunchKernelGGL((streams_kernel<T, S, 2, 256, 8>), dim3(M), dim3(256), 0, s, p);
  else hipLaunchKernelGGL((streams_kernel<T, S, 1, 1024, 8>), dim3(M), dim3(1024), 0, s, p);
  LLJ_CHECK_LAUNCH();
  return 0;
}

template <typename T>
static int streams_run(const StreamsParams& p, int M, bool vec, hipStream_t s) {
  if (vec) switch (p.S) {
      case 1: return streams_wide<T, 1>(p, M, s);
      case 2: return streams_wide<T, 2>(p, M, s);
      case 3: return streams_wide<T, 3>(p, M, s);
      case 4: return streams_wide<T, 4>(p, M, s);
    }
  const size_t lds = ((size_t)p.C + (size_t)p.S * 256) * 4;
  if (lds > 128 * 1024) return LLJ_EINVAL;
  auto kern = streams_any_kernel<T>;
  static bool attr_set = false;
  if (!attr_set) {
    hipError_t e = hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, 128 * 1024);
    if (e != hipSuccess) return (int)e;
    attr_set = true;
  }
  hipLaunchKernelGGL(kern, dim3(M), dim3(256), lds, s, p);
  LLJ_CHECK_LAUNCH();
  return 0;
}

static int streams_check(const StreamsParams& p, int M, int dt, hipStream_t s) {
  LLJ_REQUIRE(p.x && p.w && p.h && M > 0 && p.S > 0 && p.C > 0 && p.ldx >= p.C && p.ldh >= p.C && (dt == 0 || dt == 1));
  const bool vec = (p.C | p.ldx | p.ldh | (p.tok ? p.lde : p.ldy)) % 8 == 0 && p.C <= 8192 &&
                   (((uintptr_t)p.x | (uintptr_t)p.w | (uintptr_t)p.h | (uintptr_t)p.embed | (uintptr_t)p.y) & 15) == 0;
  return dt == 0 ? streams_run<bf16_t>(p, M, vec, s) : streams_run<float>(p, M, vec, s);
}

}  // namespace llj

using namespace llj;

extern "C" {
LLJ_TRACE_EXPORT(streams)

int llj_streams_embed(const int* tok, const void* embed, int lde, float scale, int* pos, float* x, int ldx, int streams,
                      const float* in, const void* norm_w, float eps, void* h, int ldh, int M, int C, int dt, void* stream) {
  LLJ_REQUIRE(tok && embed && lde >= C);
  StreamsParams p{};
  p.tok = tok; p.embed = embed; p.lde = lde; p.scale = scale; p.pos = pos;
  p.x = x; p.ldx = ldx; p.in = in; p.w = norm_w; p.eps = eps; p.h = h; p.ldh = ldh; p.S = streams; p.C = C;
  return streams_check(p, M, dt, (hipStream_t)stream);
}

int llj_streams_step(const void* y, int ldy, const float* out, const float* mix, float* x, int ldx, int streams,
                     const float* in, const void* norm_w, float eps, void* h, int ldh, const int* rows, int M, int C, int dt,
                     void* stream) {
  LLJ_REQUIRE(y && out && mix && ldy >= C);
  StreamsParams p{};
  p.y = y; p.ldy = ldy; p.out = out; p.mix = mix;
  p.x = x; p.ldx = ldx; p.in = in; p.w = norm_w; p.eps = eps; p.h = h; p.ldh = ldh; p.rows = rows; p.S = streams; p.C = C;
  return streams_check(p, M, dt, (hipStream_t)stream);
}

}  // extern "C"
