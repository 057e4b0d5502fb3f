// Decode products of hybrid models with bf16 weights (N, K): few activation rows (M <= 16), each
// weight read once and fed straight from its registers to the MFMA units.
//
// A workgroup owns 16 output columns; its NW waves take the 128-deep K chunks round robin, D chunks in
// flight per wave (a chunk of a column is 256 contiguous bytes, 16 B per lane and MFMA step), and their
// partial tiles are summed through LDS. Activation rows:
//   plain   read as MFMA fragments from memory (L2) next to the weights: no staging, no barrier before
//           the stream; lanes of rows past M read row 0 and their results are dropped;
//   post    one row (M = 1) that is the fp32 residual after a sublayer: x' = x + t / rms(t) * (1 + w) is formed
//           by every workgroup in its prologue (its operands are loaded ahead of the weight stream, which
//           then covers the reduction), rounded to bf16 as the product's input, and written once to x';
//   streams one row (M = 1) whose residual is S <= 4 fp32 streams: the update after a sublayer, the mixed row and
//           its layer norm (streams.hip) formed the same way, the new streams written once to x'.
// Few columns (N / 16 workgroups would leave CUs idle): HALF forms take 8 columns per workgroup and up to 8 rows
// and put the two halves of K side by side in the MFMA tile -- operand rows 0-7 / columns 0-7 the first
// half, rows 8-15 / columns 8-15 the second; the two diagonal quarters of the result are added.
// Output bf16, plus a bias, optionally max(., 0)^2 or the clamped gated unit of interleaved columns (elem.h).
#include "common.h"
#include "elem.h"
#include "lit_llama_amd.h"

namespace llj {

struct PostGemvParams {
  const bf16_t* A;  // plain: rows, stride lda
  int lda;
  const bf16_t* t;  // post: sublayer output (C), norm weight (C), residual in / out (C)
  const bf16_t* w;
  const float* x;
  float* xo;
  float eps;
  int C;
  const bf16_t* W;  // (N, K)
  bf16_t* out;
  int ldo, M, N, K;
  const float* bias;  // (N) or NULL
  float limit, alpha;  // clamped gated unit
  const float* so;  // streams: output weights (S), mix (S, S), input weights (S); x, xo: S rows of stride ldx
  const float* sm;
  const float* si;
  int S, ldx;
};

constexpr int kStreamsMax = 4;

// NV: post / streams: 8-column vectors per thread that cover C (0: plain)
template <int NW, int D, int NV, int ACT, bool HALF, bool STREAMS>
__global__ __launch_bounds__(NW * 64) void post_gemv_kernel(PostGemvParams p) {
  constexpr bool POST = NV > 0;  // the row comes from LDS
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  float* red = reinterpret_cast<float*>(smem);            // [NW][64][4]
  float* rs = red + NW * 256;                             // [2][NW]
  bf16_t* As = reinterpret_cast<bf16_t*>(rs + 16);        // post, streams: the row (K)
  const int tid = threadIdx.x, lane = tid & 63, wave = uniform(tid >> 6);
  const int row = lane & 15, g = lane >> 4;
  constexpr int CW = HALF ? 8 : 16;
  const int K = p.K, KC = HALF ? K >> 8 : K >> 7, n0 = blockIdx.x * CW;
  const int rc = HALF ? row & 7 : row, koff = HALF && row >= 8 ? K >> 1 : 0;  // column / row of the lane, its K half
  const u32x4* wp = reinterpret_cast<const u32x4*>(p.W + (size_t)(n0 + rc) * K + koff + 8 * g);
  const u32x4* ap = POST ? nullptr : reinterpret_cast<const u32x4*>(p.A + (size_t)(rc < p.M ? rc : 0) * p.lda + koff + 8 * g);
  u32x4 wr[D][4], ar[POST ? 1 : D][4];
  auto load = [&](int d, int i) {
    int c = wave + NW * i;
    c = c < KC ? c : KC - 1;  // past the end: a valid chunk, not used
#pragma unroll
    for (int s = 0; s < 4; ++s) {
      if constexpr (!POST) ar[d][s] = ap[(size_t)c * 16 + 4 * s];
      wr[d][s] = __builtin_nontemporal_load(wp + (size_t)c * 16 + 4 * s);
    }
  };
  const int n = KC > wave ? (KC - wave + NW - 1) / NW : 0;
  if constexpr (STREAMS) {
    u32x4 tv[NV], gv[NV];
    float xv[NV][kStreamsMax][8], u[NV][8];
#pragma unroll
    for (int v = 0; v < NV; ++v) {
      const int k = 8 * (tid + NW * 64 * v), kk = k < p.C ? k : 0;
      tv[v] = *reinterpret_cast<const u32x4*>(p.t + kk);
      gv[v] = *reinterpret_cast<const u32x4*>(p.w + kk);
#pragma unroll
      for (int s = 0; s < kStreamsMax; ++s) ld8(p.x + (size_t)(s < p.S ? s : 0) * p.ldx + kk, xv[v][s]);  // (past S: a copy)
    }
#pragma unroll
    for (int d = 0; d < D; ++d) load(d, d);
    float sum = 0.f;
#pragma unroll
    for (int v = 0; v < NV; ++v) {
      const int k = 8 * (tid + NW * 64 * v);
      const bool mine = k < p.C && (unsigned)(k >> 3) % gridDim.x == blockIdx.x;
#pragma unroll
      for (int e = 0; e < 8; ++e) u[v][e] = 0.f;
#pragma unroll
      for (int t = 0; t < kStreamsMax; ++t) {
        if (t < p.S) {  // (uniform)
          float n[8];
          const float ot = p.so[t], in = p.si ? p.si[t] : 1.f;
#pragma unroll
          for (int e = 0; e < 8; ++e) n[e] = ot * ((e & 1) ? bfhi(tv[v][e >> 1]) : bflo(tv[v][e >> 1]));
#pragma unroll
          for (int s = 0; s < kStreamsMax; ++s) {
            const float a = s < p.S ? p.sm[s * p.S + t] : 0.f;
#pragma unroll
            for (int e = 0; e < 8; ++e) n[e] += a * xv[v][s][e];
          }
          if (mine) st8(p.xo + (size_t)t * p.ldx + k, n);
#pragma unroll
          for (int e = 0; e < 8; ++e) u[v][e] += in * n[e];
        }
      }
#pragma unroll
      for (int e = 0; e < 8; ++e) sum += k < p.C ? u[v][e] : 0.f;
    }
    sum = wave_sum(sum);
    if (lane == 0) rs[wave] = sum;
    __syncthreads();
    float tot = 0.f;
#pragma unroll
    for (int i = 0; i < NW; ++i) tot += rs[i];
    const float mean = tot / (float)p.C;
    sum = 0.f;
#pragma unroll
    for (int v = 0; v < NV; ++v)
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        u[v][e] -= mean;
        sum += 8 * (tid + NW * 64 * v) < p.C ? u[v][e] * u[v][e] : 0.f;
      }
    sum = wave_sum(sum);
    if (lane == 0) rs[NW + wave] = sum;
    __syncthreads();
    tot = 0.f;
#pragma unroll
    for (int i = 0; i < NW; ++i) tot += rs[NW + i];
    const float r = 1.f / sqrtf(tot / (float)p.C + p.eps);
#pragma unroll
    for (int v = 0; v < NV; ++v) {
      const int k = 8 * (tid + NW * 64 * v);
      if (k < K) {
#pragma unroll
        for (int e = 0; e < 8; ++e)
          u[v][e] = k < p.C ? u[v][e] * r * ((e & 1) ? bfhi(gv[v][e >> 1]) : bflo(gv[v][e >> 1])) : 0.f;
        st8(As + k, u[v]);
      }
    }
    for (int k = 8 * (tid + NW * 64 * NV); k < K; k += 8 * NW * 64)
      *reinterpret_cast<uint4*>(As + k) = make_uint4(0u, 0u, 0u, 0u);
    __syncthreads();
  } else if constexpr (POST) {
    u32x4 tv[NV], gv[NV];
    float xv[NV][8];
#pragma unroll
    for (int v = 0; v < NV; ++v) {
      const int k = 8 * (tid + NW * 64 * v), kk = k < p.C ? k : 0;
      tv[v] = *reinterpret_cast<const u32x4*>(p.t + kk);
      gv[v] = *reinterpret_cast<const u32x4*>(p.w + kk);
      ld8(p.x + kk, xv[v]);
    }
#pragma unroll
    for (int d = 0; d < D; ++d) load(d, d);
    float ss = 0.f;
#pragma unroll
    for (int v = 0; v < NV; ++v) {
      if (8 * (tid + NW * 64 * v) < p.C) {
#pragma unroll
        for (int e = 0; e < 4; ++e) ss += bflo(tv[v][e]) * bflo(tv[v][e]) + bfhi(tv[v][e]) * bfhi(tv[v][e]);
      }
    }
    ss = wave_sum(ss);
    if (lane == 0) rs[wave] = ss;
    __syncthreads();
    float tot = 0.f;
#pragma unroll
    for (int i = 0; i < NW; ++i) tot += rs[i];
    const float r = 1.f / sqrtf(tot / (float)p.C + p.eps);
#pragma unroll
    for (int v = 0; v < NV; ++v) {
      const int k = 8 * (tid + NW * 64 * v);
      if (k < K) {
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          const float tt = (e & 1) ? bfhi(tv[v][e >> 1]) : bflo(tv[v][e >> 1]);
          const float gg = (e & 1) ? bfhi(gv[v][e >> 1]) : bflo(gv[v][e >> 1]);
          xv[v][e] = k < p.C ? xv[v][e] + tt * r * (1.f + gg) : 0.f;
        }
        st8(As + k, xv[v]);
        if (k < p.C && (unsigned)(k >> 3) % gridDim.x == blockIdx.x) st8(p.xo + k, xv[v]);
      }
    }
    for (int k = 8 * (tid + NW * 64 * NV); k < K; k += 8 * NW * 64)  // K's padding past the vectors
      *reinterpret_cast<uint4*>(As + k) = make_uint4(0u, 0u, 0u, 0u);
    __syncthreads();
  } else {
#pragma unroll
    for (int d = 0; d < D; ++d) load(d, d);
  }
  f32x4 acc = {0.f, 0.f, 0.f, 0.f};
  for (int i0 = 0; i0 < n; i0 += D) {
#pragma unroll
    for (int d = 0; d < D; ++d) {
      const int i = i0 + d;
      if (i < n) {  // (uniform)
#pragma unroll
        for (int s = 0; s < 4; ++s) {
          u32x4 a;
          if constexpr (POST) a = *reinterpret_cast<const u32x4*>(As + koff + 128 * (wave + NW * i) + 32 * s + 8 * g);
          else a = ar[d][s];
          acc = mfma_bf16(__builtin_bit_cast(bf16x8, a), __builtin_bit_cast(bf16x8, wr[d][s]), acc);
        }
        if (i + D < n) load(d, i + D);
      }
    }
  }
  // lane: rows 4 g + r, column n0 + row
  *reinterpret_cast<f32x4*>(red + (wave * 64 + lane) * 4) = acc;
  __syncthreads();
  auto column = [&](int m, int c) {
    float y = 0.f;
#pragma unroll
    for (int w = 0; w < NW; ++w) {
      y += red[(w * 64 + (m >> 2) * 16 + c) * 4 + (m & 3)];
      if (HALF) y += red[(w * 64 + ((m + 8) >> 2) * 16 + c + 8) * 4 + (m & 3)];
    }
    if (ACT != 1) y += p.bias ? p.bias[n0 + c] : 0.f;
    return y;
  };
  constexpr int OW = ACT == 2 ? CW / 2 : CW;  // output columns
  for (int i = tid; i < p.M * OW; i += NW * 64) {
    const int m = i / OW, c = i % OW;
    float y;
    if constexpr (ACT == 2) {
      y = clamped_glu(column(m, 2 * c), column(m, 2 * c + 1), p.limit, p.alpha);
    } else {
      y = column(m, c);
      if (ACT == 1) y = fmaxf(y, 0.f) * fmaxf(y, 0.f);
    }
    p.out[(size_t)m * p.ldo + (ACT == 2 ? n0 / 2 : n0) + c] = f2bf(y);
  }
}

template <int NW, int D, int NV, bool HALF, bool STREAMS>
static int post_gemv_go(const PostGemvParams& p, int act, hipStream_t s) {
  const size_t lds = (size_t)(NW * 256 + 16) * 4 + (NV > 0 ? (size_t)p.K * 2 : 0);
  if (lds > 64 * 1024) return LLJ_EINVAL;
  const dim3 grid(p.N / (HALF ? 8 : 16)), nt(NW * 64);
  if (act == 2) hipLaunchKernelGGL((post_gemv_kernel<NW, D, NV, 2, HALF, STREAMS>), grid, nt, lds, s, p);
  else if (act == 1 && STREAMS) return LLJ_EINVAL;
  else if (act) hipLaunchKernelGGL((post_gemv_kernel<NW, D, NV, STREAMS ? 0 : 1, HALF, STREAMS>), grid, nt, lds, s, p);
  else hipLaunchKernelGGL((post_gemv_kernel<NW, D, NV, 0, HALF, STREAMS>), grid, nt, lds, s, p);
  LLJ_CHECK_LAUNCH();
  return 0;
}

#ifndef LLJ_PG_HALF_M
#define LLJ_PG_HALF_M 8  // largest row count that takes the half-K form where it applies (A/B; 0: never)
#endif
static int post_threads(int K) { return K > 4096 ? 512 : 256; }

template <int NV, bool STREAMS = false>
static int post_gemv_launch(const PostGemvParams& p, int act, hipStream_t s) {
  const bool half = p.M <= LLJ_PG_HALF_M && p.N / 16 < 256 && p.K % 256 == 0 && p.K >= 1024;
  if constexpr (NV > 0) {  // (the thread count is post_threads')
    if (post_threads(p.K) == 512)
      return half ? post_gemv_go<8, 4, NV, true, STREAMS>(p, act, s) : post_gemv_go<8, 4, NV, false, STREAMS>(p, act, s);
    return half ? post_gemv_go<4, 4, NV, true, STREAMS>(p, act, s) : post_gemv_go<4, 4, NV, false, STREAMS>(p, act, s);
  } else {
    // waves: 8 for long K, so that a wave's chunks stay within a few rounds of the D in flight
    if (half)
      return p.K > 4096 ? post_gemv_go<8, 5, 0, true, false>(p, act, s) : post_gemv_go<4, 4, 0, true, false>(p, act, s);
    return p.K > 2048 ? post_gemv_go<8, 4, 0, false, false>(p, act, s) : post_gemv_go<4, 4, 0, false, false>(p, act, s);
  }
}

}  // namespace llj

using namespace llj;

extern "C" {
LLJ_TRACE_EXPORT(post_gemv)

int llj_rows_linear(int act, const void* A, int lda, const void* W, const float* bias, void* out, int ldo, int M, int N, int K,
                    float limit, float alpha, void* stream) {
  LLJ_REQUIRE(act >= 0 && act <= 2 && (act != 1 || !bias) && A && W && out && M >= 1 && M <= 16 && N > 0 && N % 16 == 0 &&
              K > 0 && K % 128 == 0 && lda >= K && (lda & 7) == 0 && ldo >= (act == 2 ? N / 2 : N) &&
              (((uintptr_t)A | (uintptr_t)W) & 15) == 0);
  PostGemvParams p{};
  p.A = (const bf16_t*)A; p.lda = lda; p.W = (const bf16_t*)W; p.out = (bf16_t*)out; p.ldo = ldo; p.M = M; p.N = N; p.K = K;
  p.bias = bias; p.limit = limit; p.alpha = alpha;
  return post_gemv_launch<0>(p, act, (hipStream_t)stream);
}

int llj_post_linear(int act, const void* t, const void* norm_w, float eps, const float* x, float* x_out, int C,
                    const void* W, void* out, int N, int K, void* stream) {
  LLJ_REQUIRE((act == 0 || act == 1) && t && norm_w && x && x_out && x != x_out && W && out && C > 0 && C % 8 == 0 &&
              C <= K && C <= 8192 && N > 0 && N % 16 == 0 && K > 0 && K % 128 == 0 &&
              (((uintptr_t)t | (uintptr_t)norm_w | (uintptr_t)x | (uintptr_t)x_out | (uintptr_t)W) & 15) == 0);
  PostGemvParams p{};
  p.t = (const bf16_t*)t; p.w = (const bf16_t*)norm_w; p.x = x; p.xo = x_out; p.eps = eps; p.C = C;
  p.W = (const bf16_t*)W; p.out = (bf16_t*)out; p.ldo = N; p.M = 1; p.N = N; p.K = K;
  hipStream_t s = (hipStream_t)stream;
  const int nt = post_threads(K), nv = (C / 8 + nt - 1) / nt;
  if (nv <= 1) return post_gemv_launch<1>(p, act, s);
  return post_gemv_launch<2>(p, act, s);  // C <= 8192 over 512 threads, C <= 4096 over 256
}

int llj_streams_linear_ok(int streams, int C) { return streams >= 1 && streams <= kStreamsMax && C % 8 == 0 && C > 0 && C <= 8192; }

int llj_streams_linear(int act, const void* y, const float* out_w, const float* mix, const float* x, float* x_out, int ldx,
                       int streams, const float* in, const void* norm_w, float eps, int C, const void* W, const float* bias,
                       void* out, int N, int K, float limit, float alpha, void* stream) {
  LLJ_REQUIRE((act == 0 || act == 2) && y && out_w && mix && x && x_out && x != x_out && in && norm_w && W && out &&
              llj_streams_linear_ok(streams, C) && C <= K && ldx >= C && ldx % 4 == 0 && N > 0 && N % 16 == 0 && K > 0 &&
              K % 128 == 0 && (((uintptr_t)y | (uintptr_t)norm_w | (uintptr_t)x | (uintptr_t)x_out | (uintptr_t)W) & 15) == 0);
  PostGemvParams p{};
  p.t = (const bf16_t*)y; p.w = (const bf16_t*)norm_w; p.x = x; p.xo = x_out; p.ldx = ldx; p.eps = eps; p.C = C;
  p.so = out_w; p.sm = mix; p.si = in; p.S = streams;
  p.W = (const bf16_t*)W; p.out = (bf16_t*)out; p.ldo = N; p.M = 1; p.N = N; p.K = K;
  p.bias = bias; p.limit = limit; p.alpha = alpha;
  hipStream_t s = (hipStream_t)stream;
  const int nt = post_threads(K), nv = (C / 8 + nt - 1) / nt;
  if (nv <= 1) return post_gemv_launch<1, true>(p, act, s);
  return post_gemv_launch<2, true>(p, act, s);
}

}  // extern "C"
