// Elementwise steps around the projections, for any width and for bf16 or fp32
// activations: the gated feed-forward product act(gate) * up (or the clamped gate) from
// one fused gate|up row, the normed powers of a feed-forward row, and the tanh soft cap of the
// logits.
#include "kgs_common.h"

namespace kgs {
namespace act {

enum { ACT_SILU = 0, ACT_GELU_TANH = 1, ACT_CLAMPED = 2 };

template <int ACT>
__device__ __forceinline__ float f(float z) {
  if constexpr (ACT == ACT_SILU) return z / (1.0f + expf(-z));
  return 0.5f * z * (1.0f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
}

template <int ACT>
__global__ __launch_bounds__(256) void mul_f32(const float* gu, float* o, int n, long ldi, long ldo, float limit) {
  const long r = blockIdx.y;
  const int c = blockIdx.x * 256 + threadIdx.x;
  if (c >= n) return;
  float g = gu[r * ldi + c], u = gu[r * ldi + n + c];
  if constexpr (ACT == ACT_CLAMPED) {
    g = fminf(g, limit);
    u = fminf(fmaxf(u, -limit), limit);
    o[r * ldo + c] = g / (1.0f + expf(-1.702f * g)) * (u + 1.0f);
  } else o[r * ldo + c] = f<ACT>(g) * u;
}

// 8 columns per thread (n % 8 == 0, 16-B rows)
template <int ACT>
__global__ __launch_bounds__(256) void mul_bf16(const unsigned short* gu, unsigned short* o, int n, long ldi, long ldo,
                                                float limit) {
  const long r = blockIdx.y;
  const int c = (blockIdx.x * 256 + threadIdx.x) * 8;
  if (c >= n) return;
  const bf16x8 g = *(const bf16x8*)(gu + r * ldi + c), u = *(const bf16x8*)(gu + r * ldi + n + c);
  float v[8];
#pragma unroll
  for (int i = 0; i < 8; ++i) {
    const float z = bf2f((unsigned short)g[i]), y = bf2f((unsigned short)u[i]);
    v[i] = ACT == ACT_CLAMPED ? gate_clamped(z, y, limit) : (ACT == ACT_GELU_TANH ? gelu_tanh(z) : f<ACT>(z)) * y;
  }
  *(bf16x8*)(o + r * ldo + c) = pack_bf16x8(v, 0);
}

// o = c0 N(z) + c1 N(z^2) + c2 N(z^3) + c3 with N(u) = u / sqrt(mean u^2 + eps), the mean over
// the row's n values; the padding up to np holds zeros. A workgroup per row; up to
// 8 POLY_NV values per thread stay in registers between the sums and the powers.
constexpr int POLY_NV = 4;
template <typename T>
struct Eight {
  T v[8];
};
__device__ __forceinline__ float value(unsigned short x) { return bf2f(x); }
__device__ __forceinline__ float value(float x) { return x; }
template <typename T>
__device__ __forceinline__ void powers(const Eight<T>& z, float (&s)[3]) {
#pragma unroll
  for (int i = 0; i < 8; ++i) {
    const float q = value(z.v[i]) * value(z.v[i]), q2 = q * q;
    s[0] += q;
    s[1] += q2;
    s[2] = __builtin_fmaf(q2, q, s[2]);
  }
}
template <typename T>
__device__ __forceinline__ void poly_store(T* o, const Eight<T>& z, const float (&f)[3], float e) {
  Eight<T> y;
#pragma unroll
  for (int i = 0; i < 8; ++i) {
    const float x = value(z.v[i]);
    const float r = __builtin_fmaf(__builtin_fmaf(__builtin_fmaf(f[2], x, f[1]), x, f[0]), x, e);
    if constexpr (sizeof(T) == 2) y.v[i] = f2bf(r);
    else y.v[i] = r;
  }
  *(Eight<T>*)o = y;
}
template <typename T>
__global__ __launch_bounds__(512) void poly_norm(const T* z, long ldz, const float* c, T* o, long ldo, int n, int np,
                                                 float eps) {
  __shared__ float part[3][8];
  const int tid = threadIdx.x, nt = blockDim.x, nc = np / 8;
  const T* zr = z + (long)blockIdx.x * ldz;
  T* orow = o + (long)blockIdx.x * ldo;
  Eight<T> x[POLY_NV];
  float s[3] = {0.f, 0.f, 0.f};
#pragma unroll
  for (int k = 0; k < POLY_NV; ++k)
    if (tid + k * nt < nc) x[k] = *(const Eight<T>*)(zr + 8 * (tid + k * nt));
#pragma unroll
  for (int k = 0; k < POLY_NV; ++k)
    if (tid + k * nt < nc) powers(x[k], s);
  for (int i = tid + POLY_NV * nt; i < nc; i += nt) powers(*(const Eight<T>*)(zr + 8 * i), s);
  for (int j = 0; j < 3; ++j) s[j] = wave_sum(s[j]);
  if (nt > 64) {
    if ((tid & 63) == 0)
      for (int j = 0; j < 3; ++j) part[j][tid >> 6] = s[j];
    __syncthreads();
    for (int j = 0; j < 3; ++j) {
      s[j] = 0.f;
      for (int i = 0; i < nt / 64; ++i) s[j] += part[j][i];
    }
  }
  float f[3];
#pragma unroll
  for (int j = 0; j < 3; ++j) f[j] = c[j] / sqrtf(s[j] / n + eps);
  const float e = c[3];
#pragma unroll
  for (int k = 0; k < POLY_NV; ++k)
    if (tid + k * nt < nc) poly_store(orow + 8 * (tid + k * nt), x[k], f, e);
  for (int i = tid + POLY_NV * nt; i < nc; i += nt) poly_store(orow + 8 * i, *(const Eight<T>*)(zr + 8 * i), f, e);
}

// logits [rows, ld] -> fp32 [rows, n]: cap * tanh(x / cap), or x with cap 0
template <typename T>
__global__ __launch_bounds__(256) void softcap(const T* x, float* o, int n, long ld, float cap) {
  const long r = blockIdx.y;
  const int c = blockIdx.x * 256 + threadIdx.x;
  if (c >= n) return;
  float v;
  if constexpr (sizeof(T) == 2) v = bf2f(x[r * ld + c]);
  else v = x[r * ld + c];
  o[r * n + c] = cap > 0.f ? cap * tanhf(v / cap) : v;
}

}  // namespace act
}  // namespace kgs

KGS_EXPORT int kgs_act_mul(const void* gu, void* o, int rows, int n, long ldi, long ldo, int act, float limit,
                           int f32, hipStream_t s) {
  using namespace kgs::act;
  if (rows <= 0 || rows > 65535 * 16 || n <= 0 || ldi < 2l * n || ldo < n) return KGS_ERR_SHAPE;
  if (act < ACT_SILU || act > ACT_CLAMPED) return KGS_ERR_ARG;
  if (!f32 && (n % 8 || ldi % 8 || ldo % 8 || (((uintptr_t)gu | (uintptr_t)o) & 15))) return KGS_ERR_ALIGN;
  const long per = 65535;
  for (long r0 = 0; r0 < rows; r0 += per) {
    const unsigned nr = (unsigned)(rows - r0 < per ? rows - r0 : per);
    if (f32) {
      auto k = act == ACT_SILU ? mul_f32<ACT_SILU> : act == ACT_CLAMPED ? mul_f32<ACT_CLAMPED> : mul_f32<ACT_GELU_TANH>;
      hipLaunchKernelGGL(k, dim3((n + 255) / 256, nr), dim3(256), 0, s, (const float*)gu + r0 * ldi,
                         (float*)o + r0 * ldo, n, ldi, ldo, limit);
    } else {
      auto k = act == ACT_SILU ? mul_bf16<ACT_SILU> : act == ACT_CLAMPED ? mul_bf16<ACT_CLAMPED> : mul_bf16<ACT_GELU_TANH>;
      hipLaunchKernelGGL(k, dim3((n / 8 + 255) / 256, nr), dim3(256), 0, s, (const unsigned short*)gu + r0 * ldi,
                         (unsigned short*)o + r0 * ldo, n, ldi, ldo, limit);
    }
  }
  return (int)hipGetLastError();
}

// z [rows, ldz], o [rows, ldo], np columns of which n count; c: four numbers
KGS_EXPORT int kgs_poly_norm(const void* z, long ldz, const void* c, void* o, long ldo, int rows, int n, int np,
                             float eps, int f32, hipStream_t s) {
  using namespace kgs::act;
  if (rows <= 0 || n <= 0 || np < n || ldz < np || ldo < np) return KGS_ERR_SHAPE;
  if (np % 8 || ldz % 8 || ldo % 8 || (((uintptr_t)z | (uintptr_t)o) & 15)) return KGS_ERR_ALIGN;
  const int nt = np / 8 >= 512 ? 512 : (np / 8 + 63) / 64 * 64;
  if (f32) hipLaunchKernelGGL(poly_norm<float>, dim3(rows), dim3(nt), 0, s, (const float*)z, ldz, (const float*)c, (float*)o, ldo, n, np, eps);
  else hipLaunchKernelGGL(poly_norm<unsigned short>, dim3(rows), dim3(nt), 0, s, (const unsigned short*)z, ldz, (const float*)c,
                          (unsigned short*)o, ldo, n, np, eps);
  return (int)hipGetLastError();
}

KGS_EXPORT int kgs_softcap(const void* x, void* o, int rows, int n, long ld, float cap, int f32, hipStream_t s) {
  using namespace kgs::act;
  if (rows <= 0 || rows > 65535 || n <= 0 || ld < n) return KGS_ERR_SHAPE;
  const dim3 grid((n + 255) / 256, rows);
  if (f32) hipLaunchKernelGGL(softcap<float>, grid, dim3(256), 0, s, (const float*)x, (float*)o, n, ld, cap);
  else hipLaunchKernelGGL(softcap<unsigned short>, grid, dim3(256), 0, s, (const unsigned short*)x, (float*)o, n, ld,
                          cap);
  return (int)hipGetLastError();
}
