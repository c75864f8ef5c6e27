// The fp32 residual of layers that norm what a sublayer puts out, not what it reads, and
// that mix neighbouring positions in front of their mixers. One launch
//   * adds a sublayer's output, divided by its root mean square and times one number:
//       x <- x + g y / sqrt(mean y^2 + eps)      (or starts x from the embedding table);
//   * makes what comes next read it: x itself, a causal convolution over time on each
//     channel added to it,
//       h_t = x_t + sum_d w[d] x_{t-d},  d = 0 .. taps - 1,
//     or its norm in front of the output projection.
//
// A portion's first rows need rows of earlier steps: a sequence's state is a ring of its
// last taps - 1 inputs, position p in entry p % (taps - 1). The launch that reads it never
// writes it: entries are written by the next launch on the residual, from the x it reads
// (`save`), so no row waits for another.
//
// One workgroup per row. It computes the taps - 1 rows before its own again instead of waiting
// for them, so the convolution needs x in two buffers (xi, xo); neighbouring rows run on one
// XCD, whose L2 then has them (measured: as fast as two rows per workgroup, faster than four or
// eight). Long convolutions and wide rows are a launch of their own (`conv`), which
// reads the rows back.
#include "kgs_common.h"

namespace kgs {
namespace postnorm {

constexpr int MAX_NT = 512, MAX_NV = 4;  // 8-column pieces per thread
constexpr int MAX_HALO = 3;              // rows that `step` computes again
constexpr int HALO_NV = 2;               // pieces per thread up to which it does

struct Args {
  const float* xi;    // [T, wp]
  float* xo;          // [T, wp]; xi itself where nothing is convolved
  const int* tokens;  // start of the residual: embed[token]; else null
  const void* embed;
  long lde;
  const void* y;      // the sublayer's output [T, ldy]
  long ldy;
  float g, eps;
  // next input: convolution (cw not null), norm times `gf` (final), else a copy
  const float* cw;    // [taps][wp]: row d the weight of x_{t-d}
  const float* cstate;  // [slots][taps - 1][wp]
  int final;
  float gf;
  float* save;        // ring that gets the last rows of xi, or null
  int taps;           // of both rings
  const int *row_seq, *row0, *n, *pos0, *slot;
  void* h;            // [T, ldh]
  long ldh;
  int T, width, wp;
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

// 8 values as they lie in memory
template <typename T>
struct Raw {
  f32x4 a, b;
  __device__ __forceinline__ void load(const float* p) { a = *(const f32x4*)p, b = *(const f32x4*)(p + 4); }
  __device__ __forceinline__ float at(int i) const { return i < 4 ? a[i & 3] : b[i & 3]; }
};
template <>
struct Raw<unsigned short> {
  bf16x8 a;
  __device__ __forceinline__ void load(const unsigned short* p) { a = *(const bf16x8*)p; }
  __device__ __forceinline__ float at(int i) const { return bf2f((unsigned short)a[i]); }
};

// sums[j] over the workgroup, in every thread
template <int R>
__device__ __forceinline__ void block_sums(float (&s)[R], float (*part)[MAX_NT / 64], int tid, int nt) {
#pragma unroll
  for (int j = 0; j < R; ++j) s[j] = wave_sum(s[j]);
  if (nt <= 64) return;
  if ((tid & 63) == 0)
#pragma unroll
    for (int j = 0; j < R; ++j) part[j][tid >> 6] = s[j];
  __syncthreads();
#pragma unroll
  for (int j = 0; j < R; ++j) {
    float x = part[j][0];
    for (int i = 1; i < nt / 64; ++i) x += part[j][i];
    s[j] = x;
  }
}

template <typename T, int NV, int HALO>
__global__ __launch_bounds__(MAX_NT) void step(Args a) {
  constexpr int R = HALO + 1;
  __shared__ float part[R][MAX_NT / 64];
  const int tid = threadIdx.x, nt = blockDim.x, nc = a.wp / 8;
  const int own = xcd_remap(blockIdx.x, gridDim.x);
  // the row's sequence, its number in this batch, position and first ring entry
  int sq = 0, i = 0, pos = 0, ring = 0;
  if (HALO > 0 || a.save) {
    sq = a.row_seq[own];
    i = own - a.row0[sq];
    pos = a.pos0[sq] + i;
    ring = a.slot[sq] * (a.taps - 1);
  }
  const int first = HALO - min(HALO, i);  // rows from `first` on are computed, the last is the own one

  Raw<T> y[R][NV];
  float ss[R];
  if (!a.tokens) {
#pragma unroll
    for (int j = 0; j < R; ++j) {
      ss[j] = 0.f;
      if (j < first) continue;
      const T* yp = (const T*)a.y + (long)(own - HALO + j) * a.ldy;
#pragma unroll
      for (int k = 0; k < NV; ++k) {
        const int c = tid + k * nt;
        if (c >= nc) continue;
        y[j][k].load(yp + 8 * c);
#pragma unroll
        for (int i = 0; i < 8; ++i) ss[j] = __builtin_fmaf(y[j][k].at(i), y[j][k].at(i), ss[j]);
      }
    }
    block_sums<R>(ss, part, tid, nt);
#pragma unroll
    for (int j = 0; j < R; ++j) ss[j] = a.g / sqrtf(ss[j] / a.width + a.eps);
  }

  float prev[HALO > 0 ? HALO : 1][NV][8];  // x of the rows before, the nearest first
  float v[NV][8];
#pragma unroll
  for (int j = 0; j < R; ++j) {
    if (j < first) continue;
    const int row = own - HALO + j;
#pragma unroll
    for (int k = 0; k < NV; ++k) {
      const int c = tid + k * nt;
      if (c >= nc) continue;
      if (a.tokens) load8((const T*)a.embed + (long)a.tokens[row] * a.lde + 8 * c, v[k]);
      else load8(a.xi + (long)row * a.wp + 8 * c, v[k]);
    }
    if (j == HALO && a.save && a.n[sq] - i < a.taps) {
      float* sp = a.save + (long)(ring + pos % (a.taps - 1)) * a.wp;
#pragma unroll
      for (int k = 0; k < NV; ++k) {
        const int c = tid + k * nt;
        if (c < nc) store8(sp + 8 * c, v[k]);
      }
    }
    if (!a.tokens) {
#pragma unroll
      for (int k = 0; k < NV; ++k)
#pragma unroll
        for (int e = 0; e < 8; ++e) v[k][e] = __builtin_fmaf(ss[j], y[j][k].at(e), v[k][e]);
    }
    if (j == HALO) {
      float fin = 0.f;
      if (HALO == 0 && a.final) {
        float s[1] = {0.f};
#pragma unroll
        for (int k = 0; k < NV; ++k)
          if (tid + k * nt < nc)
#pragma unroll
            for (int e = 0; e < 8; ++e) s[0] = __builtin_fmaf(v[k][e], v[k][e], s[0]);
        __syncthreads();  // the first sums are used
        block_sums<1>(s, part, tid, nt);
        fin = a.gf / sqrtf(s[0] / a.width + a.eps);
      }
#pragma unroll
      for (int k = 0; k < NV; ++k) {
        const int c = tid + k * nt;
        if (c >= nc) continue;
        store8(a.xo + (long)row * a.wp + 8 * c, v[k]);
        float o[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) o[e] = HALO == 0 && a.final ? v[k][e] * fin : v[k][e];
        if (a.cw) {
          float w[8];
          load8(a.cw + 8 * c, w);
#pragma unroll
          for (int e = 0; e < 8; ++e) o[e] = __builtin_fmaf(w[e], v[k][e], o[e]);
#pragma unroll
          for (int d = 1; d <= HALO; ++d) {
            if (pos < d) continue;  // uniform
            float u[8];
            if (i >= d) {
#pragma unroll
              for (int e = 0; e < 8; ++e) u[e] = prev[d - 1][k][e];
            } else load8(a.cstate + (long)(ring + (pos - d) % (a.taps - 1)) * a.wp + 8 * c, u);
            load8(a.cw + (long)d * a.wp + 8 * c, w);
#pragma unroll
            for (int e = 0; e < 8; ++e) o[e] = __builtin_fmaf(w[e], u[e], o[e]);
          }
        }
        store8((T*)a.h + (long)row * a.ldh + 8 * c, o);
      }
    }
    if (j < HALO) {
#pragma unroll
      for (int k = 0; k < NV; ++k)
#pragma unroll
        for (int e = 0; e < 8; ++e) prev[HALO - 1 - j][k][e] = v[k][e];
    }
  }
}

// h = x + its convolution, x complete: a workgroup per row
template <typename T>
__global__ __launch_bounds__(256) void conv(Args a) {
  const int row = blockIdx.x, c = blockIdx.y * 256 + threadIdx.x;
  if (c >= a.wp / 8) return;
  const int sq = a.row_seq[row], i = row - a.row0[sq], pos = a.pos0[sq] + i, ring = a.slot[sq] * (a.taps - 1);
  float x[8], o[8], w[8], u[8];
  load8(a.xi + (long)row * a.wp + 8 * c, x);
  load8(a.cw + 8 * c, w);
#pragma unroll
  for (int e = 0; e < 8; ++e) o[e] = __builtin_fmaf(w[e], x[e], x[e]);
  for (int d = 1; d < min(a.taps, pos + 1); ++d) {
    load8(i >= d ? a.xi + (long)(row - d) * a.wp + 8 * c
                 : a.cstate + (long)(ring + (pos - d) % (a.taps - 1)) * a.wp + 8 * c, u);
    load8(a.cw + (long)d * a.wp + 8 * c, w);
#pragma unroll
    for (int e = 0; e < 8; ++e) o[e] = __builtin_fmaf(w[e], u[e], o[e]);
  }
  store8((T*)a.h + (long)row * a.ldh + 8 * c, o);
}

int threads(const Args& a) { return a.wp / 8 >= MAX_NT ? MAX_NT : (a.wp / 8 + 63) / 64 * 64; }
int pieces(const Args& a) { return (a.wp / 8 + threads(a) - 1) / threads(a); }

template <typename T>
int launch(const Args& a, int halo, hipStream_t s) {
  static_assert(MAX_HALO == 3 && HALO_NV == 2 && MAX_NV == 4, "the instances below");
  const bool one = pieces(a) <= 1;
  auto fn = halo == 1 ? (one ? step<T, 1, 1> : step<T, 2, 1>) : halo == 2 ? (one ? step<T, 1, 2> : step<T, 2, 2>)
            : halo == 3 ? (one ? step<T, 1, 3> : step<T, 2, 3>)
                        : one ? step<T, 1, 0> : pieces(a) <= 2 ? step<T, 2, 0> : step<T, 4, 0>;
  hipLaunchKernelGGL(fn, dim3(a.T), dim3(threads(a)), 0, s, a);
  return (int)hipGetLastError();
}

}  // namespace postnorm
}  // namespace kgs

// x [T, wp] fp32: xo = xi + g y / rms(y) (tokens null), or embed[token]; then h [T, ldh]: xo,
// its norm times gf (final), or xo plus its convolution (cw [taps][wp], row d the weight of
// the row d before). A convolution of 2 to 4 taps and rows of up to 8192 columns in one launch
// (xi and xo different buffers); others in two.
// cstate, save: rings [slots][taps - 1][wp]; row_seq [T], row0 / n / pos0 / slot per sequence.
KGS_EXPORT int kgs_postnorm(const void* xi, void* xo, const void* tokens, const void* embed, long lde, const void* y,
                            long ldy, float g, float eps, const void* cw, const void* cstate, int taps, int final,
                            float gf, void* save, const void* row_seq, const void* row0, const void* n, const void* pos0,
                            const void* slot, void* h, long ldh, int T, int width, int wp, int f32, hipStream_t s) {
  using namespace kgs::postnorm;
  if (T <= 0 || width <= 0 || wp < width || wp > MAX_NT * 8 * MAX_NV || ldh < wp || taps < 1) return KGS_ERR_SHAPE;
  if (tokens ? (!embed || lde < wp || save) : (!xi || !y || ldy < wp)) return KGS_ERR_SHAPE;
  if ((cw && final) || (cw && taps > 1 && (xi == xo || !cstate)) || (save && taps < 2) ||
      ((save || (cw && taps > 1)) && (!row_seq || !row0 || !n || !pos0 || !slot)))
    return KGS_ERR_ARG;
  if (wp % 8 || ldh % 8 || (tokens ? lde : ldy) % 8 ||
      (((uintptr_t)xi | (uintptr_t)xo | (uintptr_t)embed | (uintptr_t)y | (uintptr_t)cw | (uintptr_t)cstate |
        (uintptr_t)save | (uintptr_t)h) & 15))
    return KGS_ERR_ALIGN;
  Args a{(const float*)xi, (float*)xo, (const int*)tokens, embed, lde, y, ldy, g, eps, (const float*)cw,
         (const float*)cstate, final, gf, (float*)save, taps, (const int*)row_seq, (const int*)row0, (const int*)n,
         (const int*)pos0, (const int*)slot, h, ldh, T, width, wp};
  const bool apart = cw && taps > 1 && (taps > MAX_HALO + 1 || pieces(a) > HALO_NV);
  if (apart) a.cw = nullptr;
  const int halo = a.cw ? taps - 1 : 0;
  if (int rc = f32 ? launch<float>(a, halo, s) : launch<unsigned short>(a, halo, s)) return rc;
  if (!apart) return KGS_OK;
  a.cw = (const float*)cw, a.xi = a.xo;
  const dim3 grid(T, (wp / 8 + 255) / 256);
  if (f32) hipLaunchKernelGGL(conv<float>, grid, dim3(256), 0, s, a);
  else hipLaunchKernelGGL(conv<unsigned short>, grid, dim3(256), 0, s, a);
  return (int)hipGetLastError();
}
