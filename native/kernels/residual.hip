// The fp32 residual between sublayers: one launch adds what a sublayer (or several at
// once) puts out -- a projection and its bias, every token's chosen experts' rows, rows
// times a number per token (a gated shared expert, experts that return their input) --
// and produces the next sublayer's normed input; another starts the residual from the
// embedding table, which the first can add again. RMS norm of the whole row or of equal
// consecutive parts, each by its own mean: x / sqrt(mean x^2 + eps) * (off + w), off 1
// for weights stored around zero. Activations bf16 or fp32.
//
// One workgroup per token. Rows are padded to a multiple of 8 columns whose weights
// and inputs are zero, so only the mean knows the true width.
#include "kgs_common.h"

namespace kgs {
namespace residual {

constexpr int MAX_NT = 512, MAX_NV = 4;  // 8-column chunks per thread
constexpr int MAX_SCALED = 2;

struct Args {
  float* x;           // [T, wp]
  const int* tokens;  // the embedding: start of the residual, or added again (else null)
  const void* embed;
  long lde;
  float scale;
  const void* a;      // mixer output [T, lda] or null, and its bias [wp] or null
  long lda;
  const float* ab;
  const void* y;      // expert rows [nslice][nrows][ldy] or null
  const int* pos;     // [T, top]: each choice's row, -1: none
  int top, y32, nslice;
  long ldy, yslice;
  const void* b[MAX_SCALED];   // further rows [T, ldb] or null, times s[t]
  const float* s[MAX_SCALED];
  long ldb[MAX_SCALED];
  const float* w;     // [wp]
  float off;
  int groups, unit;   // parts of the norm; columns summed by one thread (8, or 1 where a part is no multiple of it)
  void* h;            // [T, ldh]
  long ldh;
  int* zero;          // counters the next launches use, cleared here
  int nzero;
  int width, wp;
  float eps;
};

__device__ __forceinline__ void load8(const float* p, float (&v)[8]) {
  const f32x4 a = *(const f32x4*)p, b = *(const f32x4*)(p + 4);
#pragma unroll
  for (int i = 0; i < 4; ++i) v[i] = a[i], v[4 + i] = b[i];
}
__device__ __forceinline__ void load8(const unsigned short* p, float (&v)[8]) {
  const bf16x8 a = *(const bf16x8*)p;
#pragma unroll
  for (int i = 0; i < 8; ++i) v[i] = bf2f((unsigned short)a[i]);
}
__device__ __forceinline__ void store8(float* p, const float (&v)[8]) {
  *(f32x4*)p = f32x4{v[0], v[1], v[2], v[3]};
  *(f32x4*)(p + 4) = f32x4{v[4], v[5], v[6], v[7]};
}
__device__ __forceinline__ void store8(unsigned short* p, const float (&v)[8]) { *(bf16x8*)p = pack_bf16x8(v, 0); }

template <typename T, int NV, bool EMBED, bool GROUPED>
__global__ __launch_bounds__(MAX_NT) void step(Args a) {
  extern __shared__ float lds[];  // GROUPED: [wp / unit] sums, [groups] factors
  const long t = blockIdx.x;
  const int tid = threadIdx.x, nt = blockDim.x, nc = a.wp / 8;
  __shared__ float part[MAX_NT / 64];
  if (blockIdx.x == 0)
    for (int i = tid; i < a.nzero; i += nt) a.zero[i] = 0;
  float v[NV][8], ss = 0.f;
  const T* again = !EMBED && a.tokens ? (const T*)a.embed + (long)a.tokens[t] * a.lde : nullptr;
  const T* src = EMBED ? (const T*)a.embed + (long)a.tokens[t] * a.lde : (const T*)a.a + t * a.lda;
#pragma unroll
  for (int k = 0; k < NV; ++k) {
    const int c = tid + k * nt;
    if (c >= nc) continue;
    float* xp = a.x + t * a.wp + 8 * c;
    if constexpr (EMBED) {
      load8(src + 8 * c, v[k]);
#pragma unroll
      for (int i = 0; i < 8; ++i) v[k][i] *= a.scale;
    } else {
      float s[8] = {};
      if (a.a) load8(src + 8 * c, s);
      if (a.ab) {
        float b[8];
        load8(a.ab + 8 * c, b);
#pragma unroll
        for (int i = 0; i < 8; ++i) s[i] += b[i];
      }
      load8(xp, v[k]);
#pragma unroll
      for (int j = 0; j < MAX_SCALED; ++j)
        if (a.b[j]) {
          float b[8];
          load8((const T*)a.b[j] + t * a.ldb[j] + 8 * c, b);
          const float f = a.s[j][t];
#pragma unroll
          for (int i = 0; i < 8; ++i) s[i] = __builtin_fmaf(f, b[i], s[i]);
        }
      // the chosen experts' rows, four choices' loads at a time
      for (int j0 = 0; j0 < a.top; j0 += 4) {
        int p[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) p[j] = j0 + j < a.top ? a.pos[t * a.top + j0 + j] : -1;
        for (int sl = 0; sl < a.nslice; ++sl) {
          float e[4][8];
#pragma unroll
          for (int j = 0; j < 4; ++j) {
            const long o = sl * a.yslice + max(p[j], 0) * a.ldy + 8 * c;
            if (a.y32) load8((const float*)a.y + o, e[j]);
            else load8((const unsigned short*)a.y + o, e[j]);
          }
#pragma unroll
          for (int j = 0; j < 4; ++j)
#pragma unroll
            for (int i = 0; i < 8; ++i) s[i] += p[j] >= 0 ? e[j][i] : 0.f;
        }
      }
#pragma unroll
      for (int i = 0; i < 8; ++i) v[k][i] += s[i];
      if (again) {
        float e[8];
        load8(again + 8 * c, e);
#pragma unroll
        for (int i = 0; i < 8; ++i) v[k][i] = __builtin_fmaf(a.scale, e[i], v[k][i]);
      }
    }
    store8(xp, v[k]);
    if constexpr (GROUPED) {
      float q = 0.f;
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        if (a.unit == 1) lds[8 * c + i] = v[k][i] * v[k][i];
        q = __builtin_fmaf(v[k][i], v[k][i], q);
      }
      if (a.unit == 8) lds[c] = q;
    } else {
#pragma unroll
      for (int i = 0; i < 8; ++i) ss = __builtin_fmaf(v[k][i], v[k][i], ss);
    }
  }
  float inv = 0.f;
  const int gs = a.width / a.groups, gu = gs / a.unit;
  float* fac = lds + a.wp / a.unit;
  if constexpr (GROUPED) {
    __syncthreads();
    for (int g = tid >> 6; g < a.groups; g += nt / 64) {
      float q = 0.f;
      for (int i = tid & 63; i < gu; i += 64) q += lds[g * gu + i];
      q = wave_sum(q);
      if ((tid & 63) == 0) fac[g] = 1.0f / sqrtf(q / gs + a.eps);
    }
    __syncthreads();
  } else {
    ss = wave_sum(ss);
    if (nt > 64) {
      if ((tid & 63) == 0) part[tid >> 6] = ss;
      __syncthreads();
      ss = part[0];
      for (int i = 1; i < nt / 64; ++i) ss += part[i];
    }
    inv = 1.0f / sqrtf(ss / a.width + a.eps);
  }
#pragma unroll
  for (int k = 0; k < NV; ++k) {
    const int c = tid + k * nt;
    if (c >= nc) continue;
    float w[8];
    load8(a.w + 8 * c, w);
    if constexpr (GROUPED) {
      if (a.unit == 8) inv = fac[min(c / gu, a.groups - 1)];
#pragma unroll
      for (int i = 0; i < 8; ++i)
        w[i] = v[k][i] * (a.unit == 8 ? inv : fac[min((8 * c + i) / gs, a.groups - 1)]) * (a.off + w[i]);
    } else {
#pragma unroll
      for (int i = 0; i < 8; ++i) w[i] = v[k][i] * inv * (a.off + w[i]);
    }
    store8((T*)a.h + t * a.ldh + 8 * c, w);
  }
}

template <typename T, bool EMBED, bool GROUPED>
int launch(const Args& a, int rows, hipStream_t s) {
  const int nc = a.wp / 8;
  const int nt = nc >= MAX_NT ? MAX_NT : (nc + 63) / 64 * 64;
  const int nv = (nc + nt - 1) / nt;
  const size_t lds = GROUPED ? (a.wp / a.unit + a.groups) * 4 : 0;
  const dim3 grid(rows), block(nt);
  if (nv <= 1) hipLaunchKernelGGL((step<T, 1, EMBED, GROUPED>), grid, block, lds, s, a);
  else if (nv <= 2) hipLaunchKernelGGL((step<T, 2, EMBED, GROUPED>), grid, block, lds, s, a);
  else hipLaunchKernelGGL((step<T, 4, EMBED, GROUPED>), grid, block, lds, s, a);
  return (int)hipGetLastError();
}
template <bool EMBED>
int launch(Args& a, int rows, int f32, hipStream_t s) {
  if (a.groups == 1) return f32 ? launch<float, EMBED, false>(a, rows, s) : launch<unsigned short, EMBED, false>(a, rows, s);
  a.unit = a.width / a.groups % 8 ? 1 : 8;
  if ((a.wp / a.unit + a.groups) * 4 > 63 * 1024) return KGS_ERR_SHAPE;
  return f32 ? launch<float, EMBED, true>(a, rows, s) : launch<unsigned short, EMBED, true>(a, rows, s);
}

int check(const Args& a, int rows, int f32) {
  if (rows <= 0 || a.width <= 0 || a.wp < a.width || a.wp > MAX_NT * 8 * MAX_NV || a.ldh < a.wp) return KGS_ERR_SHAPE;
  if (a.groups <= 0 || a.width % a.groups) return KGS_ERR_SHAPE;
  if (a.embed && (a.lde < a.wp || !a.tokens)) return KGS_ERR_SHAPE;
  if (a.embed && (a.lde % 8 || ((uintptr_t)a.embed & 15))) return KGS_ERR_ALIGN;
  if (a.wp % 8 || a.ldh % 8 || (((uintptr_t)a.x | (uintptr_t)a.h | (uintptr_t)a.w) & 15)) return KGS_ERR_ALIGN;
  return KGS_OK;
}

}  // namespace residual
}  // namespace kgs

// x [T, wp] fp32 = scale * embed[token]; h = norm(x) in `groups` parts, weight off + w.
// zero: counters to clear, or null.
KGS_EXPORT int kgs_residual_embed(void* x, const void* tokens, const void* embed, long lde, float scale, const void* w,
                                  void* h, long ldh, void* zero, int nzero, int rows, int width, int wp, int groups,
                                  float off, float eps, int f32, hipStream_t s) {
  using namespace kgs::residual;
  Args a{};
  a.x = (float*)x, a.tokens = (const int*)tokens, a.embed = embed, a.lde = lde, a.scale = scale;
  a.w = (const float*)w, a.h = h, a.ldh = ldh, a.zero = (int*)zero, a.nzero = zero ? nzero : 0;
  a.width = width, a.wp = wp, a.eps = eps, a.groups = groups, a.unit = 8, a.off = off;
  if (!embed) return KGS_ERR_ARG;
  if (int rc = check(a, rows, f32)) return rc;
  return launch<true>(a, rows, f32, s);
}

// x += a + ab + sum of each token's expert rows y[pos[t][j]] (over nslice partial
// products, yslice elements apart) + s0[t] b0[t] + s1[t] b1[t] + scale embed[token];
// h = norm(x). Null: not there.
KGS_EXPORT int kgs_residual_add(void* x, const void* a_, long lda, const void* ab, const void* y, long ldy, long yslice,
                                int nslice, int y32, const void* pos, int top, const void* b0, long ldb0, const void* s0,
                                const void* b1, long ldb1, const void* s1, const void* tokens, const void* embed,
                                long lde, float scale, const void* w, void* h, long ldh, void* zero, int nzero,
                                int rows, int width, int wp, int groups, float off, float eps, int f32, hipStream_t s) {
  using namespace kgs::residual;
  Args a{};
  a.x = (float*)x, a.a = a_, a.lda = lda, a.ab = (const float*)ab;
  a.y = y, a.ldy = ldy, a.yslice = yslice, a.nslice = nslice, a.y32 = y32, a.pos = (const int*)pos, a.top = y ? top : 0;
  a.b[0] = b0, a.ldb[0] = ldb0, a.s[0] = (const float*)s0, a.b[1] = b1, a.ldb[1] = ldb1, a.s[1] = (const float*)s1;
  a.tokens = embed ? (const int*)tokens : nullptr, a.embed = embed, a.lde = lde, a.scale = scale;
  a.w = (const float*)w, a.h = h, a.ldh = ldh, a.zero = (int*)zero, a.nzero = zero ? nzero : 0;
  a.width = width, a.wp = wp, a.eps = eps, a.groups = groups, a.unit = 8, a.off = off;
  if (int rc = check(a, rows, f32)) return rc;
  if ((a_ && lda < wp) || (y && (ldy < wp || top <= 0 || nslice <= 0 || !pos))) return KGS_ERR_SHAPE;
  for (int j = 0; j < MAX_SCALED; ++j)
    if (a.b[j] && (a.ldb[j] < wp || !a.s[j])) return KGS_ERR_SHAPE;
  if (lda % 8 || ldy % 8 || yslice % 8 || ldb0 % 8 || ldb1 % 8 ||
      (((uintptr_t)a_ | (uintptr_t)y | (uintptr_t)ab | (uintptr_t)b0 | (uintptr_t)b1) & 15))
    return KGS_ERR_ALIGN;
  return launch<false>(a, rows, f32, s);
}
