// Grouped-query attention over per-sequence K / V rows, any mixture of prompt rows and decode rows. A cache row
// of one token is [k of every K / V head | v of every K / V head], stride ldc, at cache[slot][position]; query head h
// reads K / V head h / (H / G).
//   rotation   rotate-half on the first RD dimensions (i with i + RD / 2), the angle formed in double precision
//              in turns per position (turns[i] = frequency / 2 pi) and reduced before the fp32 sine and cosine
//   norm       queries and keys divided by their root mean square after the rotation (optional)
//   values     copied beside the cache (first, no lam) or mixed with such a copy, (1 - lam) v + lam first
//   sink       one is added to the softmax's denominator: a key of score 0 without a value (optional)
//   gate       head h's output times sigmoid(in[og + h]) (optional, og >= 0)
// Kernels: row preparation, any-size attention rows (both types), flash prefill and split decode (bf16, MFMA). The
// decode kernel prepares its own queries and the new key and value. Scores, softmax statistics and weights are
// fp32; the weights enter the MFMA product as two bf16 terms (p = hi + lo).
#include "common.h"
#include "elem.h"
#include "lit_llama_amd.h"

namespace llj {

typedef short s16x4 __attribute__((ext_vector_type(4)));

struct GqaParams {
  void* in;  // activation rows: queries at oq, keys at ok, values at ov, gates at og (-1: none)
  int ld, oq, ok, ov, og;
  const double* turns;
  int RD, qk_norm;
  float eps;
  const int* pos;      // position of each row
  const int* row_seq;  // NULL: row m is sequence m
  const int* slot;
  void* cache;  // [slots][W][ldc]
  int W, ldc;
  void* first;  // [M][ldf]
  const float* lam;
  int ldf;
  void* y;
  int ldy, M, H, G, D, V, sink;
  float scale;
};

// device-scope accesses of the decode hand-off, two floats each
__device__ __forceinline__ void put2(float* p, float a, float b) {
  const unsigned long long v = (unsigned long long)__float_as_uint(a) | ((unsigned long long)__float_as_uint(b) << 32);
  __hip_atomic_store(reinterpret_cast<unsigned long long*>(p), v, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
}
__device__ __forceinline__ float2 get2(const float* p) {
  const unsigned long long v = __hip_atomic_load(reinterpret_cast<const unsigned long long*>(p), __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
  return make_float2(__uint_as_float((uint32_t)v), __uint_as_float((uint32_t)(v >> 32)));
}

__device__ __forceinline__ void turn_cs(const double* __restrict__ turns, int i, int pos, float& c, float& s) {
  const double t = (double)pos * turns[i];
  sincospif(2.f * (float)(t - rint(t)), &s, &c);
}

__device__ __forceinline__ float group_sum(float v, int lanes) {
  for (int d = lanes >> 1; d; d >>= 1) v += __shfl_xor(v, d, 64);
  return v;
}

// One row per workgroup: rotation and norm of its queries (in place) and keys (into the cache row), its values. LG
// lanes share a head; an item is a rotated pair (i, i + RD / 2) or an unrotated dimension (VEC: 8 of them, one item
// per lane), and belongs to one lane, so the queries' update in place reads nothing another lane writes.
template <typename T, bool VEC>
__global__ __launch_bounds__(256) void gqa_prep_kernel(GqaParams p, int LG) {
  extern __shared__ __attribute__((aligned(16))) float s_cs[];  // [RD / 2] cosines, sines
  const int m = blockIdx.x, tid = threadIdx.x, n = p.RD / 2, D = p.D;
  T* row = (T*)p.in + (size_t)m * p.ld;
  const int ps = p.pos[m], b = p.row_seq ? p.row_seq[m] : m;
  T* dst = (T*)p.cache + ((size_t)p.slot[b] * p.W + ps) * p.ldc;
  for (int i = tid; i < n; i += 256) turn_cs(p.turns, i, ps, s_cs[i], s_cs[n + i]);
  __syncthreads();
  const int l = tid & (LG - 1), per = 256 / LG;
  constexpr int E = VEC ? 8 : 1;
  const int np = n / E, items = np + (D - p.RD) / E;
  for (int h = tid / LG; h < (p.H + p.G + per - 1) / per * per; h += per) {  // (uniform trip count: shuffles below)
    const bool live = h < p.H + p.G;
    const bool key = h >= p.H;
    const T* src = row + (key ? p.ok + (live ? h - p.H : 0) * D : p.oq + h * D);
    T* out = key ? dst + (live ? h - p.H : 0) * D : row + p.oq + h * D;
    auto item = [&](int it, float (&a)[E], float (&c)[E]) {  // the values at k, k + n (a pair) or at k
      const bool pair = it < np;
      const int k = pair ? E * it : p.RD + E * (it - np);
      if constexpr (VEC) {
        ld8(src + k, a);
        if (pair) ld8(src + k + n, c);
      } else {
        a[0] = ldv(src, k);
        if (pair) c[0] = ldv(src, k + n);
      }
      if (pair) {
#pragma unroll
        for (int e = 0; e < E; ++e) {
          const float cs = s_cs[k + e], sn = s_cs[n + k + e], u = a[e], v = c[e];
          a[e] = u * cs - v * sn;
          c[e] = v * cs + u * sn;
        }
      }
      return k;
    };
    float ss = 0.f, a[E] = {}, c[E] = {};
    for (int it = l; live && it < items; it += LG) {
      item(it, a, c);
#pragma unroll
      for (int e = 0; e < E; ++e) ss += a[e] * a[e] + (it < np ? c[e] * c[e] : 0.f);
    }
    ss = group_sum(ss, LG);
    const float r = p.qk_norm ? 1.f / sqrtf(ss / (float)D + p.eps) : 1.f;
    for (int it = l; live && it < items; it += LG) {
      int k = it < np ? E * it : p.RD + E * (it - np);
      if (!VEC || items > LG) k = item(it, a, c);  // (VEC: still in registers)
#pragma unroll
      for (int e = 0; e < E; ++e) {
        a[e] *= r;
        c[e] *= r;
      }
      if constexpr (VEC) {
        st8(out + k, a);
        if (it < np) st8(out + k + n, c);
      } else {
        stv(out, k, a[0]);
        if (it < np) stv(out, k + n, c[0]);
      }
    }
  }
  const int GV = p.G * p.V;
  T* vd = dst + p.G * D;
  T* fr = p.first ? (T*)p.first + (size_t)m * p.ldf : nullptr;
  const float lam = p.lam ? *p.lam : 0.f;
  for (int k = tid; k < GV; k += 256) {
    float v = ldv(row, p.ov + k);
    if (p.lam) v = (1.f - lam) * v + lam * ldv(fr, k);
    else if (fr) stv(fr, k, v);
    stv(vd, k, v);
  }
}

// Any sizes, one workgroup per (row, head): tiles of 256 keys with a running softmax.
template <typename T>
__global__ __launch_bounds__(256) void gqa_rows_kernel(GqaParams p) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  const int m = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int D = p.D, V = p.V, g = h / (p.H / p.G);
  float* s_q = sm;         // [D]
  float* s_o = s_q + D;    // [V]
  float* s_p = s_o + V;    // [256]
  float* red = s_p + 256;  // [4]
  const int b = p.row_seq ? p.row_seq[m] : m, ps = p.pos[m];
  const T* row = (const T*)p.in + (size_t)m * p.ld;
  const T* kb = (const T*)p.cache + (size_t)p.slot[b] * p.W * p.ldc + g * D;
  const T* vb = kb - g * D + p.G * D + g * V;
  for (int i = tid; i < D; i += 256) s_q[i] = ldv(row, p.oq + h * D + i);
  for (int i = tid; i < V; i += 256) s_o[i] = 0.f;
  __syncthreads();
  // (the sink is the first key: score 0, no value)
  float mx = p.sink ? 0.f : -INFINITY, l = p.sink ? 1.f : 0.f;
  for (int jt = 0; jt <= ps; jt += 256) {
    const int n = ps + 1 - jt < 256 ? ps + 1 - jt : 256;
    for (int j = wave; j < n; j += 4) {
      const T* kr = kb + (size_t)(jt + j) * p.ldc;
      float a = 0.f;
      for (int r = lane; r < D; r += 64) a += s_q[r] * ldv(kr, r);
      a = wave_sum(a) * p.scale;
      if (lane == 0) s_p[j] = a;
    }
    __syncthreads();
    const float sc = tid < n ? s_p[tid] : -INFINITY;
    float tm = wave_max(sc);
    if (lane == 0) red[wave] = tm;
    __syncthreads();
    tm = fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3]));
    const float mn = fmaxf(mx, tm), corr = expf(mx - mn);
    const float e = tid < n ? expf(sc - mn) : 0.f;
    s_p[tid] = e;
    const float ts = wave_sum(e);
    __syncthreads();
    if (lane == 0) red[wave] = ts;
    __syncthreads();
    l = l * corr + red[0] + red[1] + red[2] + red[3];
    mx = mn;
    for (int r = tid; r < V; r += 256) {
      float a = s_o[r] * corr;
      for (int j = 0; j < n; ++j) a += s_p[j] * ldv(vb + (size_t)(jt + j) * p.ldc, r);
      s_o[r] = a;
    }
    __syncthreads();
  }
  float f = 1.f / l;
  if (p.og >= 0) f /= 1.f + expf(-ldv(row, p.og + h));
  for (int r = tid; r < V; r += 256) stv((T*)p.y, (size_t)m * p.ldy + h * V + r, s_o[r] * f);
}

// ------------------------------------------------------------------------------------------ flash prefill
// One workgroup per (work item, head): 64 QB queries of one sequence, then (second half of the item) the short block
// paired with it, so that the causal triangle is spread evenly. Everything transposed: S^T = K Q^T with the wave's
// queries in registers, P^T straight from the accumulators into O^T = V^T P^T; 64-key tiles of the cache staged
// through LDS, the next one in flight in registers.
// KT: 32-deep steps of a key, DB: 16-column blocks of a value, QB: 16-query blocks per wave
template <int KT, int DB, int QB>
__global__ __launch_bounds__(256, 2) void gqa_flash_kernel(GqaParams p, const int* __restrict__ work, float sl2) {
  constexpr int KP = KT * 32 + 8, VP = DB * 16 + 16;
  extern __shared__ __attribute__((aligned(16))) bf16_t lds[];
  bf16_t* Ks = lds;            // [64][KP]
  bf16_t* Vs = lds + 64 * KP;  // [64][VP]
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, col = lane & 15, g = lane >> 4;
  // workgroups go round robin over the 8 XCDs: each takes neighbouring heads, which share K / V heads in its L2
  const int h = p.H % 8 ? blockIdx.x : (blockIdx.x & 7) * (p.H >> 3) + (blockIdx.x >> 3);
  const int gh = h / (p.H / p.G);
  const u32x4 zero = {0, 0, 0, 0};
  for (int part = 0; part < 2; ++part) {
    const int r0 = work[6 * blockIdx.y + 3 * part], n = work[6 * blockIdx.y + 3 * part + 1], b = work[6 * blockIdx.y + 3 * part + 2];
    if (n <= 0) break;
    if (part) __syncthreads();  // the first block's last readers are done
    const int plo = p.pos[r0], phi = plo + n - 1;
    const bf16_t* kb = (const bf16_t*)p.cache + (size_t)p.slot[b] * p.W * p.ldc + gh * p.D;
    const bf16_t* vb = kb - gh * p.D + p.G * p.D + gh * p.V;
    int t[QB], qpos[QB];
    u32x4 qf[QB][KT];
#pragma unroll
    for (int qi = 0; qi < QB; ++qi) {
      t[qi] = (wave * QB + qi) * 16 + col;
      const int tq = t[qi] < n ? t[qi] : n - 1;  // rows past the block: a copy, never stored
      qpos[qi] = plo + tq;
      const bf16_t* qrow = (const bf16_t*)p.in + (size_t)(r0 + tq) * p.ld + p.oq + h * p.D;
#pragma unroll
      for (int kk = 0; kk < KT; ++kk) {
        const int c = 32 * kk + 8 * g;
        qf[qi][kk] = c < p.D ? *reinterpret_cast<const u32x4*>(qrow + c) : zero;
      }
    }
    const int ntile = phi / 64 + 1;
    constexpr int PK = 64 * KT * 4 / 256, PV = 64 * DB * 2 / 256;
    u32x4 kr[PK], vr[PV];
    auto load = [&](int kt) {
#pragma unroll
      for (int i = 0; i < PK; ++i) {
        const int piece = tid + 256 * i, c = 8 * (piece % (KT * 4));
        int j = 64 * kt + piece / (KT * 4);
        j = j < phi ? j : phi;  // clamped: masked below
        const u32x4 x = *reinterpret_cast<const u32x4*>(kb + (size_t)j * p.ldc + (c < p.D ? c : 0));
        kr[i] = c < p.D ? x : zero;
      }
#pragma unroll
      for (int i = 0; i < PV; ++i) {
        const int piece = tid + 256 * i, c = 8 * (piece % (DB * 2));
        int j = 64 * kt + piece / (DB * 2);
        j = j < phi ? j : phi;
        const u32x4 x = *reinterpret_cast<const u32x4*>(vb + (size_t)j * p.ldc + (c < p.V ? c : 0));
        vr[i] = c < p.V ? x : zero;
      }
    };
    float m_run[QB], l_run[QB];
    f32x4 acc[QB][DB];
#pragma unroll
    for (int qi = 0; qi < QB; ++qi) {
      m_run[qi] = p.sink ? 0.f : -INFINITY;  // (the sink is the first key: score 0, no value)
      l_run[qi] = p.sink ? 1.f : 0.f;
#pragma unroll
      for (int d = 0; d < DB; ++d) acc[qi][d] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
    load(0);
    for (int kt = 0; kt < ntile; ++kt) {
      __syncthreads();  // the previous tile's readers are done
#pragma unroll
      for (int i = 0; i < PK; ++i) {
        const int piece = tid + 256 * i;
        *reinterpret_cast<u32x4*>(Ks + (piece / (KT * 4)) * KP + 8 * (piece % (KT * 4))) = kr[i];
      }
#pragma unroll
      for (int i = 0; i < PV; ++i) {
        const int piece = tid + 256 * i;
        *reinterpret_cast<u32x4*>(Vs + (piece / (DB * 2)) * VP + 8 * (piece % (DB * 2))) = vr[i];
      }
      __syncthreads();
      if (kt + 1 < ntile) load(kt + 1);  // in flight during this tile's MFMAs
      f32x4 s[QB][4];
#pragma unroll
      for (int j = 0; j < 4; ++j) {
#pragma unroll
        for (int qi = 0; qi < QB; ++qi) s[qi][j] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int kk = 0; kk < KT; ++kk) {
          const bf16x8 a = __builtin_bit_cast(bf16x8, *reinterpret_cast<const u32x4*>(Ks + (16 * j + col) * KP + 32 * kk + 8 * g));
#pragma unroll
          for (int qi = 0; qi < QB; ++qi) s[qi][j] = mfma_bf16(a, __builtin_bit_cast(bf16x8, qf[qi][kk]), s[qi][j]);
        }
      }
      uint32_t ph[QB][4][2], pl[QB][4][2];
      // only tiles that reach past the wave's first query cross the diagonal (uniform)
      const bool masked = 64 * kt + 63 > plo + wave * 16 * QB;
#pragma unroll
      for (int qi = 0; qi < QB; ++qi) {
        float mx = -INFINITY;
#pragma unroll
        for (int j = 0; j < 4; ++j)
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            s[qi][j][r] *= sl2;
            if (masked) s[qi][j][r] = 64 * kt + 16 * j + 4 * g + r <= qpos[qi] ? s[qi][j][r] : -INFINITY;
            mx = fmaxf(mx, s[qi][j][r]);
          }
        {
          float a, c;
          lane_halves<false>(mx, a, c);
          mx = fmaxf(a, c);
          lane_halves<true>(mx, a, c);
          mx = fmaxf(a, c);
        }
        const float m_new = fmaxf(m_run[qi], mx);  // finite: key 0 is visible to every query
        const float corr = __builtin_amdgcn_exp2f(m_run[qi] - m_new);
        float psum = 0.f;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          float pr[4], lo[4];
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            pr[r] = __builtin_amdgcn_exp2f(s[qi][j][r] - m_new);
            psum += pr[r];
            lo[r] = pr[r] - round_bf(pr[r]);
          }
          ph[qi][j][0] = pack2bf(pr[0], pr[1]);
          ph[qi][j][1] = pack2bf(pr[2], pr[3]);
          pl[qi][j][0] = pack2bf(lo[0], lo[1]);
          pl[qi][j][1] = pack2bf(lo[2], lo[3]);
        }
        {
          float a, c;
          lane_halves<false>(psum, a, c);
          psum = a + c;
          lane_halves<true>(psum, a, c);
          psum = a + c;
        }
        l_run[qi] = l_run[qi] * corr + psum;
        m_run[qi] = m_new;
        if (__any(corr != 1.f)) {
#pragma unroll
          for (int d = 0; d < DB; ++d)
#pragma unroll
            for (int r = 0; r < 4; ++r) acc[qi][d][r] *= corr;
        }
      }
#pragma unroll
      for (int u = 0; u < 2; ++u) {
#pragma unroll
        for (int d = 0; d < DB; ++d) {
          // transposing LDS read: lane receives column 16 d + col of keys 32 u + 4 g + 0 .. 3 (and + 16)
          const bf16_t* va = Vs + (32 * u + 4 * g + ((lane >> 2) & 3)) * VP + 16 * d + 4 * (lane & 3);
          const s16x4 a = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s16x4*)va);
          const s16x4 c = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s16x4*)(va + 16 * VP));
          const uint2 a2 = __builtin_bit_cast(uint2, a), c2 = __builtin_bit_cast(uint2, c);
          const bf16x8 av = __builtin_bit_cast(bf16x8, u32x4{a2.x, a2.y, c2.x, c2.y});
#pragma unroll
          for (int qi = 0; qi < QB; ++qi) {
            const u32x4 bh = {ph[qi][2 * u][0], ph[qi][2 * u][1], ph[qi][2 * u + 1][0], ph[qi][2 * u + 1][1]};
            const u32x4 bl = {pl[qi][2 * u][0], pl[qi][2 * u][1], pl[qi][2 * u + 1][0], pl[qi][2 * u + 1][1]};
            acc[qi][d] = mfma_bf16(av, __builtin_bit_cast(bf16x8, bh), acc[qi][d]);
            acc[qi][d] = mfma_bf16(av, __builtin_bit_cast(bf16x8, bl), acc[qi][d]);
          }
        }
      }
    }
#pragma unroll
    for (int qi = 0; qi < QB; ++qi)
      if (t[qi] < n) {  // lane holds columns 16 d + 4 g + r of its query
        float f = 1.f / l_run[qi];
        if (p.og >= 0) f /= 1.f + __expf(-bf2f(((const bf16_t*)p.in)[(size_t)(r0 + t[qi]) * p.ld + p.og + h]));
        bf16_t* yr = (bf16_t*)p.y + (size_t)(r0 + t[qi]) * p.ldy + h * p.V;
#pragma unroll
        for (int d = 0; d < DB; ++d) {
          const int v = 16 * d + 4 * g;
          if (v < p.V)
            *reinterpret_cast<uint2*>(yr + v) = make_uint2(pack2bf(acc[qi][d][0] * f, acc[qi][d][1] * f), pack2bf(acc[qi][d][2] * f, acc[qi][d][3] * f));
        }
      }
  }
}

// ------------------------------------------------------------------------------------------ split decode
// One workgroup per (key range, K / V head and up to 16 of its query heads, row). Prologue: the heads' queries rotated and
// normed into LDS; the range that ends with the row's own position also prepares that key and value, stores
// them in the cache and takes them from LDS. The waves then walk 32-key steps of the range on their own (no
// barriers): K fragments straight from the cache, S^T = K q^T, P from the accumulators, V through a wave's LDS
// tile and transposing reads. The waves' results are merged through LDS; one range: the result itself, else fp32 partials
// [M][H][nsplit][VW + 4] (o unnormalized, then max in log2 units, sum), which the last of the ranges' workgroups to
// finish merges in range order. The hand-off: device-scope (write-through) stores, a wait for them, one device-scope
// counter per (row, heads), device-scope loads; nobody waits for another workgroup, and the last one resets the counter.
__host__ __device__ constexpr size_t gqa_attend_lds(int KT, int DB, int n) {
  return (size_t)(17 * (KT * 32 + 8) + DB * 16) * 2 + (size_t)4 * 32 * (DB * 16 + 16) * 2 + (size_t)2 * n * 4 + 2 * 64 * 4;
}

template <int KT, int DB>
__global__ __launch_bounds__(256) void gqa_attend_kernel(GqaParams p, float* partials, int* count, int nsplit, float sl2) {
  constexpr int KW = KT * 32, QP = KW + 8, VW = DB * 16, VP = VW + 16;
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  bf16_t* Qs = reinterpret_cast<bf16_t*>(smem);  // [16][QP] queries, then the new key
  bf16_t* Kn = Qs + 16 * QP;
  bf16_t* Vn = Kn + QP;                          // [VW] the new value
  bf16_t* Vs = Vn + VW;                          // [4][32][VP]
  float* cs = reinterpret_cast<float*>(Vs + 4 * 32 * VP);  // cosines, sines
  const int n = p.RD / 2;
  float* wm = cs + 2 * n;  // [4][16] the waves' maxima, sums
  float* wl = wm + 64;
  const int R = p.H / p.G, HB = (R + 15) / 16;
  const int sp = blockIdx.x, gh = blockIdx.y / HB, hb = blockIdx.y % HB, m = blockIdx.z;
  const int h0 = gh * R + 16 * hb, nh = R - 16 * hb < 16 ? R - 16 * hb : 16;
  const int tid = threadIdx.x, lane = tid & 63, wave = uniform(tid >> 6), col = lane & 15, g = lane >> 4;
  const int ps = p.pos[m], D = p.D, V = p.V;
  const int steps = ps / 32 + 1, per = (steps + nsplit - 1) / nsplit;
  const int s0 = sp * per, s1 = s0 + per < steps ? s0 + per : steps;
  const bool owner = s0 < s1 && s1 == steps;
  bf16_t* kb = (bf16_t*)p.cache + (size_t)p.slot[m] * p.W * p.ldc + gh * D;
  bf16_t* vb = kb - gh * D + p.G * D + gh * V;
  const u32x4 zero = {0, 0, 0, 0};
  u32x4 kf[2][KT], vr[DB];
  // (padding columns and keys past the position read a valid place; masked or multiplied by zeros)
  auto fetch = [&](int t) {
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      const int key = 32 * t + 16 * j + col;
      const bf16_t* kr = kb + (size_t)(key < ps ? key : ps) * p.ldc;
#pragma unroll
      for (int kk = 0; kk < KT; ++kk) {
        const int c = 32 * kk + 8 * g;
        kf[j][kk] = *reinterpret_cast<const u32x4*>(kr + (c < D ? c : 0));
      }
    }
#pragma unroll
    for (int i = 0; i < DB; ++i) {
      const int piece = lane + 64 * i, key = 32 * t + piece / (2 * DB), c = 8 * (piece % (2 * DB));
      vr[i] = *reinterpret_cast<const u32x4*>(vb + (size_t)(key < ps ? key : ps) * p.ldc + (c < V ? c : 0));
    }
  };
  // ---- queries and the new key: 16 lanes per head; their loads first (a lane's items as in the preparation kernel: pairs,
  // then unrotated dimensions), then the first step's keys and values, all in flight over the angles
  const bf16_t* row = (const bf16_t*)p.in + (size_t)m * p.ld;
  constexpr int NI = 2 * KT;  // items per lane, at most
  const int hh = tid >> 4, l = tid & 15, items = n + D - p.RD;
  const bool qlive = hh < nh;
  bf16_t qa[NI], qc[NI], ka[NI], kc[NI];
  auto place = [&](int j, int& k, bool& pair) {  // (items past the end read a valid place and are dropped)
    const int it = l + 16 * j;
    pair = it < n;
    k = pair ? it : p.RD + it - n;
    const bool in = it < items;
    k = in ? k : 0;
    return in;
  };
  {
    const bf16_t* qs = row + p.oq + (h0 + (qlive ? hh : 0)) * D;
    const bf16_t* ks = row + p.ok + gh * D;
#pragma unroll
    for (int j = 0; j < NI; ++j) {
      int k;
      bool pair;
      place(j, k, pair);
      qa[j] = qs[k];
      qc[j] = qs[pair ? k + n : k];
      ka[j] = ks[k];
      kc[j] = ks[pair ? k + n : k];
    }
  }
  if (s0 + wave < s1) fetch(s0 + wave);
  for (int i = tid; i < n; i += 256) turn_cs(p.turns, i, ps, cs[i], cs[n + i]);
  for (int i = tid; i < 17 * QP / 8; i += 256) *reinterpret_cast<u32x4*>(Qs + 8 * i) = zero;
  __syncthreads();
  auto prepare = [&](const bf16_t (&a)[NI], const bf16_t (&c)[NI], bool live, bf16_t* out, bf16_t* out2) {
    float u[NI], v[NI], ss = 0.f;
#pragma unroll
    for (int j = 0; j < NI; ++j) {
      int k;
      bool pair;
      const bool in = place(j, k, pair);
      u[j] = bf2f(a[j]);
      v[j] = 0.f;
      if (pair) {
        const float x = u[j], y = bf2f(c[j]), co = cs[k], si = cs[n + k];
        u[j] = x * co - y * si;
        v[j] = y * co + x * si;
      }
      ss += in ? u[j] * u[j] + v[j] * v[j] : 0.f;
    }
    ss = row16_sum(ss);
    const float r = p.qk_norm ? 1.f / sqrtf(ss / (float)D + p.eps) : 1.f;
#pragma unroll
    for (int j = 0; j < NI; ++j) {
      int k;
      bool pair;
      if (place(j, k, pair) && live) {
        const bf16_t x = f2bf(u[j] * r), y = f2bf(v[j] * r);
        out[k] = x;
        if (pair) out[k + n] = y;
        if (out2) {
          out2[k] = x;
          if (pair) out2[k + n] = y;
        }
      }
    }
  };
  prepare(qa, qc, qlive, Qs + hh * QP, nullptr);
  if (owner && wave == 0) prepare(ka, kc, hh == 0, Kn, kb + (size_t)ps * p.ldc);
  if (owner && tid < VW) {
    bf16_t o = 0;
    if (tid < V) {
      float v = bf2f(row[p.ov + gh * V + tid]);
      bf16_t* fr = p.first ? (bf16_t*)p.first + (size_t)m * p.ldf + gh * V + tid : nullptr;
      if (p.lam) v = (1.f - *p.lam) * v + *p.lam * bf2f(*fr);
      else if (fr) *fr = f2bf(v);
      o = f2bf(v);
      vb[(size_t)ps * p.ldc + tid] = o;
    }
    Vn[tid] = o;
  }
  __syncthreads();
  u32x4 qf[KT];
#pragma unroll
  for (int kk = 0; kk < KT; ++kk) qf[kk] = *reinterpret_cast<const u32x4*>(Qs + col * QP + 32 * kk + 8 * g);
  bf16_t* Vw = Vs + wave * 32 * VP;
  float m_run = -INFINITY, l_run = 0.f;  // of head col (the same in the four lane groups)
  f32x4 acc[DB];
#pragma unroll
  for (int d = 0; d < DB; ++d) acc[d] = f32x4{0.f, 0.f, 0.f, 0.f};
  for (int t = s0 + wave; t < s1; t += 4) {
    const bool last = owner && t == steps - 1;  // (uniform) holds the new key
    f32x4 s[2];
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      s[j] = f32x4{0.f, 0.f, 0.f, 0.f};
      const bool fresh = last && 32 * t + 16 * j + col >= ps;
#pragma unroll
      for (int kk = 0; kk < KT; ++kk) {
        const int c = 32 * kk + 8 * g;
        u32x4 a = c < D ? kf[j][kk] : zero;
        if (last) {
          const u32x4 x = *reinterpret_cast<const u32x4*>(Kn + c);
          a = fresh ? x : a;
        }
        s[j] = mfma_bf16(__builtin_bit_cast(bf16x8, a), __builtin_bit_cast(bf16x8, qf[kk]), s[j]);
      }
    }
#pragma unroll
    for (int i = 0; i < DB; ++i) {
      const int piece = lane + 64 * i, key = piece / (2 * DB), c = 8 * (piece % (2 * DB));
      u32x4 a = c < V ? vr[i] : zero;
      if (last) {
        const u32x4 x = *reinterpret_cast<const u32x4*>(Vn + c);
        a = 32 * t + key >= ps ? x : a;
      }
      *reinterpret_cast<u32x4*>(Vw + key * VP + c) = a;
    }
    if (t + 4 < s1) fetch(t + 4);  // in flight over this step's products
    float mx = -INFINITY;
#pragma unroll
    for (int j = 0; j < 2; ++j)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        s[j][r] = 32 * t + 16 * j + 4 * g + r <= ps ? s[j][r] * sl2 : -INFINITY;
        mx = fmaxf(mx, s[j][r]);
      }
    {
      float a, b;
      lane_halves<false>(mx, a, b);
      mx = fmaxf(a, b);
      lane_halves<true>(mx, a, b);
      mx = fmaxf(a, b);
    }
    const float m_new = fmaxf(m_run, mx);  // finite: a step's first key is visible
    const float corr = __builtin_amdgcn_exp2f(m_run - m_new);
    float ls = 0.f;
    uint32_t ph[4], pl[4];
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      float pr[4], lo[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        pr[r] = __builtin_amdgcn_exp2f(s[j][r] - m_new);
        ls += pr[r];
        lo[r] = pr[r] - round_bf(pr[r]);
      }
      ph[2 * j] = pack2bf(pr[0], pr[1]);
      ph[2 * j + 1] = pack2bf(pr[2], pr[3]);
      pl[2 * j] = pack2bf(lo[0], lo[1]);
      pl[2 * j + 1] = pack2bf(lo[2], lo[3]);
    }
    {
      float a, b;
      lane_halves<false>(ls, a, b);
      ls = a + b;
      lane_halves<true>(ls, a, b);
      ls = a + b;
    }
    l_run = l_run * corr + ls;
    m_run = m_new;
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");  // the wave's V tile is written (its LDS accesses are in order)
    __builtin_amdgcn_wave_barrier();
    const bf16x8 bh = __builtin_bit_cast(bf16x8, u32x4{ph[0], ph[1], ph[2], ph[3]});
    const bf16x8 bl = __builtin_bit_cast(bf16x8, u32x4{pl[0], pl[1], pl[2], pl[3]});
#pragma unroll
    for (int d = 0; d < DB; ++d) {
#pragma unroll
      for (int r = 0; r < 4; ++r) acc[d][r] *= corr;
      const bf16_t* va = Vw + (4 * g + ((lane >> 2) & 3)) * VP + 16 * d + 4 * (lane & 3);
      const s16x4 a = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s16x4*)va);
      const s16x4 c = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s16x4*)(va + 16 * VP));
      const uint2 a2 = __builtin_bit_cast(uint2, a), c2 = __builtin_bit_cast(uint2, c);
      const bf16x8 av = __builtin_bit_cast(bf16x8, u32x4{a2.x, a2.y, c2.x, c2.y});
      acc[d] = mfma_bf16(av, bh, acc[d]);
      acc[d] = mfma_bf16(av, bl, acc[d]);
    }
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");  // ... and read, before the next step's writes
    __builtin_amdgcn_wave_barrier();
  }
  __syncthreads();
  // ---- the four waves' results, in order
  constexpr int RP = VW + 4;
  float* red = reinterpret_cast<float*>(Vs);  // [4][16][RP]
#pragma unroll
  for (int d = 0; d < DB; ++d) *reinterpret_cast<f32x4*>(red + (wave * 16 + col) * RP + 16 * d + 4 * g) = acc[d];
  if (g == 0) {
    wm[wave * 16 + col] = m_run;
    wl[wave * 16 + col] = l_run;
  }
  __syncthreads();
  for (int i = tid; i < nh * (VW / 4); i += 256) {
    const int hh = i / (VW / 4), v = 4 * (i % (VW / 4));
    const float mx = fmaxf(fmaxf(wm[hh], wm[16 + hh]), fmaxf(wm[32 + hh], wm[48 + hh]));
    const float mu = mx == -INFINITY ? 0.f : mx;  // a range without keys: every weight exp2(-inf) = 0
    float l = 0.f;
    f32x4 o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int w = 0; w < 4; ++w) {
      const float e = __builtin_amdgcn_exp2f(wm[16 * w + hh] - mu);
      l += e * wl[16 * w + hh];
      o += *reinterpret_cast<const f32x4*>(red + (w * 16 + hh) * RP + v) * e;
    }
    if (nsplit == 1) {
      const float mt = p.sink ? fmaxf(mx, 0.f) : mx, e = __builtin_amdgcn_exp2f(mx - mt);
      float f = e / (e * l + (p.sink ? __builtin_amdgcn_exp2f(-mt) : 0.f));
      if (p.og >= 0) f /= 1.f + __expf(-bf2f(row[p.og + h0 + hh]));
      bf16_t* yr = (bf16_t*)p.y + (size_t)m * p.ldy + (h0 + hh) * V + v;
      if (v < V) *reinterpret_cast<uint2*>(yr) = make_uint2(pack2bf(o[0] * f, o[1] * f), pack2bf(o[2] * f, o[3] * f));
    } else {
      float* dst = partials + (((size_t)m * p.H + h0 + hh) * nsplit + sp) * RP;
      put2(dst + v, o[0], o[1]);
      put2(dst + v + 2, o[2], o[3]);
      if (v == 0) put2(dst + VW, mx, l);
    }
  }
  if (nsplit == 1) return;
  // ---- the last of the ranges' workgroups merges them
  asm volatile("s_waitcnt vmcnt(0)" ::: "memory");  // this wave's partials are out
  __syncthreads();
  int* last = reinterpret_cast<int*>(wm);
  if (tid == 0) {
    int* c = count + (size_t)m * gridDim.y + blockIdx.y;
    const int done = __hip_atomic_fetch_add(c, 1, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
    *last = done == nsplit - 1;
    if (done == nsplit - 1) __hip_atomic_store(c, 0, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
  }
  __syncthreads();
  if (!*last) return;
  const float* part = partials + ((size_t)m * p.H + h0) * nsplit * RP;
  float* sw = red;  // [nh][64] the ranges' weights (the waves' results are used up)
  float2 a[8], b[8];
  auto pieces = [&](int i, int s0) {  // 4 columns of 8 ranges (past the end: a copy, dropped)
    const float* q = part + (size_t)(i / (VW / 4)) * nsplit * RP + 4 * (i % (VW / 4));
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      const float* r = q + (size_t)(s0 + e < nsplit ? s0 + e : nsplit - 1) * RP;
      a[e] = get2(r);
      b[e] = get2(r + 2);
    }
  };
  const int tot = nh * (VW / 4);
  if (tid < tot) pieces(tid, 0);  // in flight over the weights
  for (int hh = wave; hh < nh; hh += 4) {  // nsplit <= 64
    float2 st = make_float2(-INFINITY, 0.f);
    if (lane < nsplit) st = get2(part + ((size_t)hh * nsplit + lane) * RP + VW);
    const float gate = p.og >= 0 ? bf2f(row[p.og + h0 + hh]) : 0.f;
    const float mt = fmaxf(wave_max(st.x), p.sink ? 0.f : -INFINITY);
    const float w = __builtin_amdgcn_exp2f(st.x - mt);
    float L = wave_sum(w * st.y) + (p.sink ? __builtin_amdgcn_exp2f(-mt) : 0.f);
    if (p.og >= 0) L *= 1.f + __expf(-gate);
    if (lane < nsplit) sw[hh * 64 + lane] = w / L;
  }
  __syncthreads();
  for (int i = tid; i < tot; i += 256) {
    const int hh = i / (VW / 4), v = 4 * (i % (VW / 4));
    f32x4 o = {0.f, 0.f, 0.f, 0.f};
    for (int s0 = 0; s0 < nsplit; s0 += 8) {
      if (i != tid || s0) pieces(i, s0);
#pragma unroll
      for (int e = 0; e < 8; ++e)
        if (s0 + e < nsplit) o += f32x4{a[e].x, a[e].y, b[e].x, b[e].y} * sw[hh * 64 + s0 + e];
    }
    bf16_t* yr = (bf16_t*)p.y + (size_t)m * p.ldy + (h0 + hh) * V + v;
    if (v < V) *reinterpret_cast<uint2*>(yr) = make_uint2(pack2bf(o[0], o[1]), pack2bf(o[2], o[3]));
  }
}

static int gqa_check(const GqaParams& p) {
  LLJ_REQUIRE(p.in && p.pos && p.slot && p.cache && p.W > 0 && p.M > 0 && p.H > 0 && p.G > 0 && p.H % p.G == 0 && p.D > 0 &&
              p.V > 0 && p.ldc >= p.G * (p.D + p.V) && p.oq >= 0 && p.oq + p.H * p.D <= p.ld &&
              (p.og < 0 || p.og + p.H <= p.ld));
  return 0;
}
static int gqa_check_new(const GqaParams& p) {
  LLJ_REQUIRE((p.turns || !p.RD) && p.RD >= 0 && p.RD % 2 == 0 && p.RD <= p.D && p.ok >= 0 && p.ok + p.G * p.D <= p.ld && p.ov >= 0 &&
              p.ov + p.G * p.V <= p.ld && (!p.lam || p.first) && (!p.first || p.ldf >= p.G * p.V));
  return 0;
}
// sizes of the MFMA kernels
static bool gqa_tiled(int dim, int vdim) { return dim > 0 && dim % 8 == 0 && dim <= 256 && vdim > 0 && vdim % 8 == 0 && vdim <= 256; }
static bool gqa_aligned(const GqaParams& p) {
  return gqa_tiled(p.D, p.V) && p.ldc % 8 == 0 && ((uintptr_t)p.cache & 15) == 0;
}

template <typename K>
static int lds_limit(K kern, size_t lds) {
  return (int)hipFuncSetAttribute((const void*)kern, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
}

template <int KT, int DB, int QB>
static int gqa_flash_go(const GqaParams& p, const int* work, int nwork, float sl2, hipStream_t s) {
  auto kern = gqa_flash_kernel<KT, DB, QB>;
  const size_t lds = (size_t)64 * (KT * 32 + 8 + DB * 16 + 16) * 2;
  static bool set = false;
  if (!set) {
    if (const int rc = lds_limit(kern, lds)) return rc;
    set = true;
  }
  hipLaunchKernelGGL(kern, dim3(p.H, nwork), dim3(256), lds, s, p, work, sl2);
  LLJ_CHECK_LAUNCH();
  return 0;
}

template <int KT, int DB>
static int gqa_attend_go(const GqaParams& p, float* part, int* count, int nsplit, float sl2, hipStream_t s) {
  auto kern = gqa_attend_kernel<KT, DB>;
  const size_t lds = gqa_attend_lds(KT, DB, p.RD / 2);
  static bool set = false;
  if (!set) {
    if (const int rc = lds_limit(kern, gqa_attend_lds(KT, DB, 16 * KT))) return rc;
    set = true;
  }
  const int R = p.H / p.G;
  hipLaunchKernelGGL(kern, dim3(nsplit, p.G * ((R + 15) / 16), p.M), dim3(256), lds, s, p, part, count, nsplit, sl2);
  LLJ_CHECK_LAUNCH();
  return 0;
}

template <int DB>
static int gqa_flash_keys(const GqaParams& p, const int* work, int nwork, int rows, float sl2, hipStream_t s) {
#define LLJ_GF(KT) (rows == 128 ? gqa_flash_go<KT, DB, 2>(p, work, nwork, sl2, s) : gqa_flash_go<KT, DB, 1>(p, work, nwork, sl2, s))
  if (p.D <= 64) return LLJ_GF(2);
  if (p.D <= 128) return LLJ_GF(4);
  if (rows == 128) return LLJ_EINVAL;
  return gqa_flash_go<8, DB, 1>(p, work, nwork, sl2, s);
#undef LLJ_GF
}

template <int DB>
static int gqa_attend_keys(const GqaParams& p, float* part, int* count, int nsplit, float sl2, hipStream_t s) {
  if (p.D <= 64) return gqa_attend_go<2, DB>(p, part, count, nsplit, sl2, s);
  if (p.D <= 128) return gqa_attend_go<4, DB>(p, part, count, nsplit, sl2, s);
  return gqa_attend_go<8, DB>(p, part, count, nsplit, sl2, s);
}

}  // namespace llj

using namespace llj;

extern "C" {
LLJ_TRACE_EXPORT(gqa)

int llj_gqa_prep(void* in, int ld, int oq, int ok, int ov, const void* turns, int rot_dims, int qk_norm, float eps,
                 const int* pos, const int* row_seq, const int* slot, void* cache, int W, int ldc, void* first,
                 const float* lam, int ldf, int M, int heads, int kv_heads, int dim, int vdim, int dt, void* stream) {
  GqaParams p{};
  p.in = in; p.ld = ld; p.oq = oq; p.ok = ok; p.ov = ov; p.og = -1;
  p.turns = (const double*)turns; p.RD = rot_dims; p.qk_norm = qk_norm; p.eps = eps;
  p.pos = pos; p.row_seq = row_seq; p.slot = slot; p.cache = cache; p.W = W; p.ldc = ldc;
  p.first = first; p.lam = lam; p.ldf = ldf; p.M = M; p.H = heads; p.G = kv_heads; p.D = dim; p.V = vdim;
  LLJ_REQUIRE(dt == 0 || dt == 1);
  if (const int rc = gqa_check(p)) return rc;
  if (const int rc = gqa_check_new(p)) return rc;
  const size_t lds = (size_t)(rot_dims > 0 ? rot_dims : 2) * 4;
  LLJ_REQUIRE(lds <= 64 * 1024);
  const int n8 = rot_dims / 16 + (dim - rot_dims) / 8;
  const bool vec = (ld | oq | ok | dim | ldc) % 8 == 0 && rot_dims % 16 == 0 && n8 <= 64 &&
                   (((uintptr_t)in | (uintptr_t)cache) & 15) == 0;
  int lg = 64;
  if (vec)
    while (lg > 1 && lg / 2 >= n8) lg /= 2;
  hipStream_t s = (hipStream_t)stream;
#define LLJ_GP(T)                                                                                          \
  do {                                                                                                     \
    if (vec) hipLaunchKernelGGL((gqa_prep_kernel<T, true>), dim3(M), dim3(256), lds, s, p, lg);            \
    else hipLaunchKernelGGL((gqa_prep_kernel<T, false>), dim3(M), dim3(256), lds, s, p, lg);               \
  } while (0)
  LLJ_DT(dt, LLJ_GP(bf16_t), LLJ_GP(float));
#undef LLJ_GP
  LLJ_CHECK_LAUNCH();
  return 0;
}

int llj_gqa_rows(const void* in, int ld, int oq, int og, const int* pos, const int* row_seq, const int* slot, const void* cache,
                 int W, int ldc, void* y, int ldy, int M, int heads, int kv_heads, int dim, int vdim, float scale, int sink,
                 int dt, void* stream) {
  GqaParams p{};
  p.in = (void*)in; p.ld = ld; p.oq = oq; p.og = og; p.pos = pos; p.row_seq = row_seq; p.slot = slot;
  p.cache = (void*)cache; p.W = W; p.ldc = ldc; p.y = y; p.ldy = ldy; p.M = M; p.H = heads; p.G = kv_heads; p.D = dim;
  p.V = vdim; p.sink = sink; p.scale = scale;
  if (const int rc = gqa_check(p)) return rc;
  const size_t lds = ((size_t)dim + vdim + 256 + 4) * 4;
  LLJ_REQUIRE(y && ldy >= heads * vdim && heads <= 65535 && lds <= 64 * 1024 && (dt == 0 || dt == 1));
  hipStream_t s = (hipStream_t)stream;
  LLJ_DT(dt, hipLaunchKernelGGL(gqa_rows_kernel<bf16_t>, dim3(M, heads), dim3(256), lds, s, p),
         hipLaunchKernelGGL(gqa_rows_kernel<float>, dim3(M, heads), dim3(256), lds, s, p));
  LLJ_CHECK_LAUNCH();
  return 0;
}

int llj_gqa_flash_rows(int dim, int vdim, int long_prompt) {
  if (!gqa_tiled(dim, vdim)) return 0;
  return long_prompt && dim <= 128 && vdim <= 128 ? 128 : 64;
}

int llj_gqa_flash(const void* in, int ld, int oq, int og, const int* work, int nwork, int rows, const int* pos, const int* slot,
                  const void* cache, int W, int ldc, void* y, int ldy, int M, int heads, int kv_heads, int dim, int vdim,
                  float scale, int sink, void* stream) {
  GqaParams p{};
  p.in = (void*)in; p.ld = ld; p.oq = oq; p.og = og; p.pos = pos; p.slot = slot; p.cache = (void*)cache; p.W = W; p.ldc = ldc;
  p.y = y; p.ldy = ldy; p.M = M; p.H = heads; p.G = kv_heads; p.D = dim; p.V = vdim; p.sink = sink; p.scale = scale;
  if (const int rc = gqa_check(p)) return rc;
  LLJ_REQUIRE(work && nwork > 0 && nwork <= 65535 && y && ldy >= heads * vdim && ldy % 4 == 0 && gqa_aligned(p) &&
              (rows == 64 || (rows == 128 && dim <= 128 && vdim <= 128)) && (ld | oq) % 8 == 0 &&
              (((uintptr_t)in | (uintptr_t)y) & 15) == 0);
  const float sl2 = scale * 1.4426950408889634f;
  hipStream_t s = (hipStream_t)stream;
  if (vdim <= 64) return gqa_flash_keys<4>(p, work, nwork, rows, sl2, s);
  if (vdim <= 128) return gqa_flash_keys<8>(p, work, nwork, rows, sl2, s);
  return gqa_flash_keys<16>(p, work, nwork, 64, sl2, s);
}

int llj_gqa_decode_ok(int dim, int vdim) { return gqa_tiled(dim, vdim); }

int llj_gqa_part_width(int vdim) { return (vdim <= 64 ? 64 : vdim <= 128 ? 128 : 256) + 4; }

int llj_gqa_decode(const void* in, int ld, int oq, int ok, int ov, int og, const void* turns, int rot_dims, int qk_norm,
                   float eps, const int* pos, const int* slot, void* cache, int W, int ldc, void* first, const float* lam,
                   int ldf, float* part, int* count, int nsplit, void* y, int ldy, int M, int heads, int kv_heads, int dim, int vdim,
                   float scale, int sink, void* stream) {
  GqaParams p{};
  p.in = (void*)in; p.ld = ld; p.oq = oq; p.ok = ok; p.ov = ov; p.og = og;
  p.turns = (const double*)turns; p.RD = rot_dims; p.qk_norm = qk_norm; p.eps = eps;
  p.pos = pos; p.slot = slot; p.cache = cache; p.W = W; p.ldc = ldc; p.first = first; p.lam = lam; p.ldf = ldf;
  p.y = y; p.ldy = ldy; p.M = M; p.H = heads; p.G = kv_heads; p.D = dim; p.V = vdim; p.sink = sink; p.scale = scale;
  if (const int rc = gqa_check(p)) return rc;
  if (const int rc = gqa_check_new(p)) return rc;
  LLJ_REQUIRE(y && ldy >= heads * vdim && ldy % 4 == 0 && gqa_aligned(p) && M <= 65535 && nsplit >= 1 && nsplit <= 64 &&
              kv_heads * ((heads / kv_heads + 15) / 16) <= 65535 && (nsplit == 1 || (part && count)) &&
              (((uintptr_t)part | (uintptr_t)y) & 15) == 0);
  const float sl2 = scale * 1.4426950408889634f;
  hipStream_t s = (hipStream_t)stream;
  if (vdim <= 64) return gqa_attend_keys<4>(p, part, count, nsplit, sl2, s);
  if (vdim <= 128) return gqa_attend_keys<8>(p, part, count, nsplit, sl2, s);
  return gqa_attend_keys<16>(p, part, count, nsplit, sl2, s);
}

}  // extern "C"
