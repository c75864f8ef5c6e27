// Hyper-connections: a token's residual is S parallel fp32 streams x_1 .. x_S
// instead of one. One launch does everything between two sublayers:
//
//   x_t <- sum_s mix[s][t] x_s + out[t] y      (write-back of the sublayer that
//                                               just ran; all streams from the
//                                               old ones)
//   u   =  sum_s in[s] x_s                     (read-out for the next one)
//   h   =  u / sqrt(mean(u^2) + eps) * w       (its pre-norm)
//
// so the streams (the largest tensor of the layer: 4 S D bytes per token) pass
// through HBM once per sublayer. `y`, `h` and the embedding are bf16 or fp32;
// the streams, the sums and the norm are fp32. With S = 1, in = mix = out = 1 it
// is the plain residual add + RMSNorm with an fp32 residual.
//
// Two sources of the streams: MODE_STEP reads them; MODE_EMBED starts them, all
// equal to rmsnorm(embed[token]) * w0. One workgroup per token; u stays in LDS
// between the sum of squares and the scaling.
#include "kgs_common.h"

namespace kgs {
namespace hyper {

constexpr int NT = 256;
constexpr int MAX_STREAMS = 8;
constexpr int MAX_WIDTH = 32768;  // u in LDS: 128 KB

enum { MODE_STEP = 0, MODE_EMBED = 1 };

struct Args {
  float* x;             // [T, S, D]
  const void* y;        // [T, ldy] or null (no write-back)
  const float* mix;     // [S, S], [from][to]
  const float* out;     // [S]
  const float* in;      // [S]
  const float* w;       // [D]
  void* h;              // [T, ldh]; columns D .. ldh are zeroed
  const int* tokens;    // MODE_EMBED
  const void* embed;    // [vocab, lde]
  const float* w0;      // [D]
  long ldy, ldh, lde;
  int D;
  float eps;
};

template <typename T>
__device__ __forceinline__ float ld(const T* p) {
  if constexpr (sizeof(T) == 2) return bf2f(*(const unsigned short*)p);
  else return *p;
}
template <typename T>
__device__ __forceinline__ void st(T* p, float v) {
  if constexpr (sizeof(T) == 2) *(unsigned short*)p = f2bf(v);
  else *p = v;
}
// 4 consecutive elements (aligned to 4 elements)
template <typename T>
__device__ __forceinline__ float4 ld4(const T* p) {
  if constexpr (sizeof(T) == 2) {
    const uint2 v = *(const uint2*)p;
    return make_float4(bf2f((unsigned short)(v.x & 0xffff)), bf2f((unsigned short)(v.x >> 16)),
                       bf2f((unsigned short)(v.y & 0xffff)), bf2f((unsigned short)(v.y >> 16)));
  } else {
    return *(const float4*)p;
  }
}
template <typename T>
__device__ __forceinline__ void st4(T* p, float4 v) {
  if constexpr (sizeof(T) == 2) {
    uint2 o;
    o.x = pack_bf16x2(v.x, v.y);
    o.y = pack_bf16x2(v.z, v.w);
    *(uint2*)p = o;
  } else {
    *(float4*)p = v;
  }
}

// sum over the workgroup, the same value in every thread; red: NT / 64 floats
__device__ __forceinline__ float block_sum(float v, float* red) {
  v = wave_sum(v);
  __syncthreads();
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  float s = 0.f;
#pragma unroll
  for (int i = 0; i < NT / 64; ++i) s += red[i];
  return s;
}

__device__ __forceinline__ float4 f4_fma(float a, float4 b, float4 c) {
  return make_float4(__builtin_fmaf(a, b.x, c.x), __builtin_fmaf(a, b.y, c.y), __builtin_fmaf(a, b.z, c.z),
                     __builtin_fmaf(a, b.w, c.w));
}
__device__ __forceinline__ float sq4(float4 v) { return v.x * v.x + v.y * v.y + v.z * v.z + v.w * v.w; }

// V: 4 elements per access (every row start and D a multiple of 4), else 1
template <typename T, int S, int MODE, int V>
__global__ __launch_bounds__(NT) void step(Args a) {
  extern __shared__ float ubuf[];  // [D]
  __shared__ float red[NT / 64];
  const int D = a.D;
  const long t = blockIdx.x;
  float* xr = a.x + t * S * D;
  float in[S], outw[S], mix[S][S];
#pragma unroll
  for (int s = 0; s < S; ++s) in[s] = a.in[s];
  const bool wb = MODE == MODE_STEP && a.y != nullptr;
  if (wb) {
#pragma unroll
    for (int s = 0; s < S; ++s) {
      outw[s] = a.out[s];
#pragma unroll
      for (int q = 0; q < S; ++q) mix[s][q] = a.mix[s * S + q];
    }
  }
  float ss = 0.f;
  if constexpr (MODE == MODE_EMBED) {
    const T* e = (const T*)a.embed + (long)a.tokens[t] * a.lde;
    for (int d = threadIdx.x * V; d < D; d += NT * V) {
      if constexpr (V == 4) ss += sq4(ld4(e + d));
      else { const float v = ld(e + d); ss += v * v; }
    }
    const float r0 = 1.0f / sqrtf(block_sum(ss, red) / D + a.eps);
    float sin = 0.f;
#pragma unroll
    for (int s = 0; s < S; ++s) sin += in[s];
    ss = 0.f;
    for (int d = threadIdx.x * V; d < D; d += NT * V) {
      if constexpr (V == 4) {
        const float4 v = ld4(e + d), w = *(const float4*)(a.w0 + d);
        const float4 n = make_float4(v.x * r0 * w.x, v.y * r0 * w.y, v.z * r0 * w.z, v.w * r0 * w.w);
#pragma unroll
        for (int s = 0; s < S; ++s) *(float4*)(xr + (long)s * D + d) = n;
        const float4 u = make_float4(sin * n.x, sin * n.y, sin * n.z, sin * n.w);
        *(float4*)(ubuf + d) = u;
        ss += sq4(u);
      } else {
        const float n = ld(e + d) * r0 * a.w0[d];
#pragma unroll
        for (int s = 0; s < S; ++s) xr[(long)s * D + d] = n;
        const float u = sin * n;
        ubuf[d] = u;
        ss += u * u;
      }
    }
  } else {
    const T* y = (const T*)a.y + t * a.ldy;
    for (int d = threadIdx.x * V; d < D; d += NT * V) {
      if constexpr (V == 4) {
        float4 x[S];
#pragma unroll
        for (int s = 0; s < S; ++s) x[s] = *(const float4*)(xr + (long)s * D + d);
        if (wb) {
          const float4 yv = ld4(y + d);
          float4 n[S];
#pragma unroll
          for (int q = 0; q < S; ++q) {
            n[q] = make_float4(outw[q] * yv.x, outw[q] * yv.y, outw[q] * yv.z, outw[q] * yv.w);
#pragma unroll
            for (int s = 0; s < S; ++s) n[q] = f4_fma(mix[s][q], x[s], n[q]);
          }
#pragma unroll
          for (int q = 0; q < S; ++q) {
            x[q] = n[q];
            *(float4*)(xr + (long)q * D + d) = n[q];
          }
        }
        float4 u = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
        for (int s = 0; s < S; ++s) u = f4_fma(in[s], x[s], u);
        *(float4*)(ubuf + d) = u;
        ss += sq4(u);
      } else {
        float x[S];
#pragma unroll
        for (int s = 0; s < S; ++s) x[s] = xr[(long)s * D + d];
        if (wb) {
          const float yv = ld(y + d);
          float n[S];
#pragma unroll
          for (int q = 0; q < S; ++q) {
            n[q] = outw[q] * yv;
#pragma unroll
            for (int s = 0; s < S; ++s) n[q] = __builtin_fmaf(mix[s][q], x[s], n[q]);
          }
#pragma unroll
          for (int q = 0; q < S; ++q) {
            x[q] = n[q];
            xr[(long)q * D + d] = n[q];
          }
        }
        float u = 0.f;
#pragma unroll
        for (int s = 0; s < S; ++s) u = __builtin_fmaf(in[s], x[s], u);
        ubuf[d] = u;
        ss += u * u;
      }
    }
  }
  const float r = 1.0f / sqrtf(block_sum(ss, red) / D + a.eps);
  T* h = (T*)a.h + t * a.ldh;
  for (int d = threadIdx.x * V; d < D; d += NT * V) {
    if constexpr (V == 4) {
      const float4 u = *(const float4*)(ubuf + d), w = *(const float4*)(a.w + d);
      st4(h + d, make_float4(u.x * r * w.x, u.y * r * w.y, u.z * r * w.z, u.w * r * w.w));
    } else {
      st(h + d, ubuf[d] * r * a.w[d]);
    }
  }
  for (int d = D + threadIdx.x; d < a.ldh; d += NT) st(h + d, 0.f);
}

template <typename T, int S, int MODE>
static hipError_t launch_v(const Args& a, int T_, hipStream_t s) {
  const uintptr_t al = (uintptr_t)a.x | (uintptr_t)a.y | (uintptr_t)a.w | (uintptr_t)a.w0 | (uintptr_t)a.h |
                       (uintptr_t)a.embed;
  const bool v4 = a.D % 4 == 0 && a.ldy % 4 == 0 && a.ldh % 4 == 0 && a.lde % 4 == 0 && (al & 15) == 0;
  const size_t lds = sizeof(float) * a.D;
  auto k = v4 ? step<T, S, MODE, 4> : step<T, S, MODE, 1>;
  if (lds > 48 * 1024) {
    const hipError_t e = hipFuncSetAttribute((const void*)k, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    if (e != hipSuccess) return e;
  }
  hipLaunchKernelGGL(k, dim3(T_), dim3(NT), lds, s, a);
  return hipGetLastError();
}

template <typename T, int MODE>
static hipError_t launch(const Args& a, int T_, int S, hipStream_t s) {
  switch (S) {
    case 1: return launch_v<T, 1, MODE>(a, T_, s);
    case 2: return launch_v<T, 2, MODE>(a, T_, s);
    case 3: return launch_v<T, 3, MODE>(a, T_, s);
    case 4: return launch_v<T, 4, MODE>(a, T_, s);
    case 5: return launch_v<T, 5, MODE>(a, T_, s);
    case 6: return launch_v<T, 6, MODE>(a, T_, s);
    case 7: return launch_v<T, 7, MODE>(a, T_, s);
    default: return launch_v<T, 8, MODE>(a, T_, s);
  }
}

}  // namespace hyper
}  // namespace kgs

// f32 != 0: y, h and embed are fp32, else bf16. y may be null (no write-back).
KGS_EXPORT int kgs_hyper_step(void* x, const void* y, const void* mix, const void* out, const void* in, const void* w,
                              void* h, int T, int S, int D, long ldy, long ldh, float eps, int f32, hipStream_t s) {
  using namespace kgs::hyper;
  if (T <= 0 || S <= 0 || S > MAX_STREAMS || D <= 0 || D > MAX_WIDTH || ldh < D || (y && ldy < D)) return KGS_ERR_SHAPE;
  Args a{(float*)x, y, (const float*)mix, (const float*)out, (const float*)in, (const float*)w, h, nullptr, nullptr,
         nullptr, y ? ldy : 0, ldh, 0, D, eps};
  return (int)(f32 ? launch<float, MODE_STEP>(a, T, S, s) : launch<unsigned short, MODE_STEP>(a, T, S, s));
}

// Streams of T tokens from their embedding rows: every stream = rmsnorm(embed[token]) * w0.
KGS_EXPORT int kgs_hyper_embed(void* x, const void* tokens, const void* embed, const void* w0, const void* in,
                               const void* w, void* h, int T, int S, int D, long lde, long ldh, float eps, int f32,
                               hipStream_t s) {
  using namespace kgs::hyper;
  if (T <= 0 || S <= 0 || S > MAX_STREAMS || D <= 0 || D > MAX_WIDTH || ldh < D || lde < D) return KGS_ERR_SHAPE;
  Args a{(float*)x, nullptr, nullptr, nullptr, (const float*)in, (const float*)w, h, (const int*)tokens, embed,
         (const float*)w0, 0, ldh, lde, D, eps};
  return (int)(f32 ? launch<float, MODE_EMBED>(a, T, S, s) : launch<unsigned short, MODE_EMBED>(a, T, S, s));
}
