// Gated delta rule with one decay per key channel: per sequence and head a
// K x V state S, for each token
//
//   S <- diag(g) S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q
//
// Sequences of a call are ragged: sequence b is rows row0[b] .. row0[b] + n[b] - 1
// at positions pos0[b] .., its state in slot[b] of the pools; pos0 = 0 starts from
// zeros whatever the slot holds, so freeing a slot needs no clear. One token per
// sequence (decode) is the n = 1 case of the same kernels.
//
//   prep   the short causal convolutions + silu of q, k, v (tail of the previous
//          portion from the pool), unit norms, log decays, step sizes;
//   scan   the recurrence and the convolution tails' update;
//   out    per-head RMS norm and output gate.
//
// Everything from prep on is fp32. K is padded to KP, a multiple of 32, in q, k,
// log g and the state (pads are zero and stay zero). The state is stored
// transposed, [slot][head][V][KP].
#include "kgs_common.h"

namespace kgs {
namespace delta {

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
__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
  for (int m = 8; m >= 1; m >>= 1) v += __shfl_xor(v, m, 64);
  return xor32_sum(xor16_sum(v));
}
__device__ __forceinline__ float sigmoid(float x) { return 1.0f / (1.0f + expf(-x)); }

struct Args {
  // inputs of prep
  const void* z;   // [T, ldz]: q (G K), k (G K), v (H V) channels at oq, ok, ov; step sizes (H) at ob
  const void* a2;  // [T, lda]: decay projection, H x K
  const float* cw;       // [taps][C] convolution weights, C = 2 G K + H V (q, k, v channels)
  const float* A_log;    // [H]
  const float* dt_bias;  // [H K]
  long ldz, lda;
  int oq, ok, ov, ob;
  int taps, G, H, K, V, KP, C;
  // ragged batch
  const int *row_seq, *row0, *n, *pos0, *slot;
  int B, T;
  // intermediates, fp32
  float *q, *k;    // [T, G, KP]
  float* v;        // [T, H, V]
  float* lg;       // [T, H, KP] log decays
  float *beta, *qk;  // [T, H], [T, G] (q . k)
  float* o;        // [T, H, V]
  // pools of this layer
  float* S;     // [slots][H][V][KP]
  float* conv;  // [slots][taps - 1][C]
};

// ----------------------------------------------------------------------- prep
// channel c (0 .. C-1) of row t after the convolution and silu
template <typename T>
__device__ __forceinline__ float conv_silu(const Args& a, long t, int c, int col, int r0, int p0, long slot) {
  float s = 0.f;
  for (int j = 0; j < a.taps; ++j) {
    const long src = t - (a.taps - 1) + j;
    float x;
    if (src >= r0) x = ld((const T*)a.z + src * a.ldz + col);
    else x = p0 > 0 ? a.conv[(slot * (a.taps - 1) + (src - r0 + a.taps - 1)) * a.C + c] : 0.f;
    s = __builtin_fmaf(a.cw[(long)j * a.C + c], x, s);
  }
  return s / (1.0f + expf(-s));
}

// one workgroup per (row, q/k head) with the value heads that read it
template <typename T>
__global__ __launch_bounds__(256) void prep(Args a) {
  extern __shared__ float buf[];  // [2][KP]
  __shared__ float red[3][4];
  const int tid = threadIdx.x;
  const long t = blockIdx.x;
  const int gh = blockIdx.y, K = a.K, KP = a.KP, V = a.V, rep = a.H / a.G;
  const int b = a.row_seq[t];
  const int r0 = a.row0[b], p0 = a.pos0[b];
  const long slot = a.slot[b];
  float sq = 0.f, sk = 0.f, sqk = 0.f;
  for (int i = tid; i < KP; i += 256) {
    float q = 0.f, k = 0.f;
    if (i < K) {
      const int c = gh * K + i;
      q = conv_silu<T>(a, t, c, a.oq + c, r0, p0, slot);
      k = conv_silu<T>(a, t, a.G * K + c, a.ok + c, r0, p0, slot);
    }
    buf[i] = q;
    buf[KP + i] = k;
    sq += q * q;
    sk += k * k;
    sqk += q * k;
  }
  sq = wave_sum(sq);
  sk = wave_sum(sk);
  sqk = wave_sum(sqk);
  if ((tid & 63) == 0) {
    red[0][tid >> 6] = sq;
    red[1][tid >> 6] = sk;
    red[2][tid >> 6] = sqk;
  }
  __syncthreads();
  sq = red[0][0] + red[0][1] + red[0][2] + red[0][3];
  sk = red[1][0] + red[1][1] + red[1][2] + red[1][3];
  sqk = red[2][0] + red[2][1] + red[2][2] + red[2][3];
  const float rq = 1.0f / sqrtf(sq + 1e-6f) / sqrtf((float)K), rk = 1.0f / sqrtf(sk + 1e-6f);
  for (int i = tid; i < KP; i += 256) {
    a.q[(t * a.G + gh) * KP + i] = buf[i] * rq;
    a.k[(t * a.G + gh) * KP + i] = buf[KP + i] * rk;
  }
  if (tid == 0) a.qk[t * a.G + gh] = sqk * rq * rk;
  for (int i = tid; i < rep * V; i += 256) {
    const int c = gh * rep * V + i;
    a.v[t * a.H * V + c] = conv_silu<T>(a, t, 2 * a.G * K + c, a.ov + c, r0, p0, slot);
  }
  for (int i = tid; i < rep * KP; i += 256) {
    const int h = gh * rep + i / KP, c = i % KP;
    float lg = 0.f;
    if (c < K) {
      const float x = ld((const T*)a.a2 + t * a.lda + h * K + c) + a.dt_bias[h * K + c];
      lg = -expf(a.A_log[h]) * (fmaxf(x, 0.f) + log1pf(expf(-fabsf(x))));
    }
    a.lg[(t * a.H + h) * KP + c] = lg;
  }
  for (int i = tid; i < rep; i += 256) {
    const int h = gh * rep + i;
    a.beta[t * a.H + h] = sigmoid(ld((const T*)a.z + t * a.ldz + a.ob + h));
  }
}

// ----------------------------------------------------------------------- scan
constexpr int TB = 8;     // tokens staged per step
constexpr int COLS = 32;  // state columns per workgroup (4 waves x 8)

__device__ __forceinline__ float xor8_sum(float x) {  // row_ror:8 within 16 lanes
  return x + __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), 0x128, 0xf, 0xf, false));
}

// The convolution tails after the call: the last taps - 1 inputs of the sequence.
template <typename T>
__device__ __forceinline__ void conv_tail(const Args& a, int b, int part, int parts) {
  const int r0 = a.row0[b], n = a.n[b], p0 = a.pos0[b], m = a.taps - 1;
  const long slot = a.slot[b];
  for (int c = part * 256 + threadIdx.x; c < a.C; c += parts * 256) {
    const int GK = a.G * a.K;
    const int col = c < GK ? a.oq + c : c < 2 * GK ? a.ok + c - GK : a.ov + c - 2 * GK;
    for (int j = 0; j < m; ++j) {  // ascending: reads are ahead of the writes
      const int src = n + j;       // index in (old tail, this portion)
      float x;
      if (src < m) x = p0 > 0 ? a.conv[(slot * m + src) * a.C + c] : 0.f;
      else x = ld((const T*)a.z + (long)(r0 + src - m) * a.ldz + col);
      a.conv[(slot * m + j) * a.C + c] = x;
    }
  }
}

// A wave owns 8 columns of one head's state: lane (rg = lane >> 3, col = lane & 7)
// holds rows 32 i + 4 rg + j of its column, so the two dot products of a token
// (with k and with q, the latter completed by (q . k) u) are one 3-step exchange.
template <typename T, int NI>
__global__ __launch_bounds__(256) void scan(Args a) {
  constexpr int KP = 32 * NI;
  __shared__ __attribute__((aligned(16))) float sq[TB][KP], sk[TB][KP], sg[TB][KP];
  __shared__ float sv[TB][COLS], sb[TB], sqk[TB];
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6;
  const int rg = lane >> 3;
  const int b = blockIdx.z, h = blockIdx.y, c0 = blockIdx.x * COLS;
  const int col = c0 + 8 * w + (lane & 7), V = a.V, H = a.H, G = a.G;
  const int gh = h / (H / G);
  const int r0 = a.row0[b], n = a.n[b];
  const bool live = col < V;
  float* Sp = a.S + (((long)a.slot[b] * H + h) * V + (live ? col : 0)) * KP + 4 * rg;
  f32x4 S[NI];
#pragma unroll
  for (int i = 0; i < NI; ++i) S[i] = a.pos0[b] > 0 && live ? *(const f32x4*)(Sp + 32 * i) : f32x4{};
  for (int t0 = 0; t0 < n; t0 += TB) {
    const int nt = min(TB, n - t0);
    __syncthreads();
    for (int i = tid; i < nt * (KP / 4); i += 256) {
      const int t = i / (KP / 4), c = 4 * (i % (KP / 4));
      const long r = r0 + t0 + t;
      *(f32x4*)&sq[t][c] = *(const f32x4*)(a.q + (r * G + gh) * KP + c);
      *(f32x4*)&sk[t][c] = *(const f32x4*)(a.k + (r * G + gh) * KP + c);
      const f32x4 g = *(const f32x4*)(a.lg + (r * H + h) * KP + c);
      *(f32x4*)&sg[t][c] = f32x4{expf(g[0]), expf(g[1]), expf(g[2]), expf(g[3])};
    }
    if (tid < nt * COLS) {
      const int t = tid / COLS, c = c0 + tid % COLS;
      sv[t][tid % COLS] = c < V ? a.v[((long)(r0 + t0 + t) * H + h) * V + c] : 0.f;
    }
    if (tid < nt) {
      sb[tid] = a.beta[(long)(r0 + t0 + tid) * H + h];
      sqk[tid] = a.qk[(long)(r0 + t0 + tid) * G + gh];
    }
    __syncthreads();
    for (int t = 0; t < nt; ++t) {
      f32x4 k[NI];
      float dk = 0.f, dq = 0.f;
#pragma unroll
      for (int i = 0; i < NI; ++i) {
        k[i] = *(const f32x4*)&sk[t][32 * i + 4 * rg];
        const f32x4 q = *(const f32x4*)&sq[t][32 * i + 4 * rg];
        const f32x4 g = *(const f32x4*)&sg[t][32 * i + 4 * rg];
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const float x = S[i][j] * g[j];
          S[i][j] = x;
          dk = __builtin_fmaf(x, k[i][j], dk);
          dq = __builtin_fmaf(x, q[j], dq);
        }
      }
      dk = xor32_sum(xor16_sum(xor8_sum(dk)));
      dq = xor32_sum(xor16_sum(xor8_sum(dq)));
      const float u = sb[t] * (sv[t][8 * w + (lane & 7)] - dk);
#pragma unroll
      for (int i = 0; i < NI; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) S[i][j] = __builtin_fmaf(k[i][j], u, S[i][j]);
      if (rg == 0 && live) a.o[((long)(r0 + t0 + t) * H + h) * V + col] = __builtin_fmaf(sqk[t], u, dq);
    }
  }
  if (live) {
#pragma unroll
    for (int i = 0; i < NI; ++i) *(f32x4*)(Sp + 32 * i) = S[i];
  }
  conv_tail<T>(a, b, h * gridDim.x + blockIdx.x, H * gridDim.x);
}

// ------------------------------------------------------------------------ out
struct OutArgs {
  const float* o;     // [T, H, V]
  const float* w;     // [V]
  const void* gate;   // [T, ldg], H x V
  void* y;            // [T, ldy], columns H V .. ldy zeroed
  long ldg, ldy;
  int H, V;
  float eps;
};

template <typename T>
__global__ __launch_bounds__(256) void out(OutArgs a) {
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
  const long t = blockIdx.x;
  const T* gate = (const T*)a.gate + t * a.ldg;
  T* y = (T*)a.y + t * a.ldy;
  for (int h = w; h < a.H; h += 4) {
    const float* o = a.o + (t * a.H + h) * a.V;
    float ss = 0.f;
    for (int i = lane; i < a.V; i += 64) ss += o[i] * o[i];
    const float r = 1.0f / sqrtf(wave_sum(ss) / a.V + a.eps);
    for (int i = lane; i < a.V; i += 64) st(y + h * a.V + i, o[i] * r * a.w[i] * sigmoid(ld(gate + h * a.V + i)));
  }
  for (int i = a.H * a.V + threadIdx.x; i < a.ldy; i += 256) st(y + i, 0.f);
}

template <typename T>
static hipError_t run_prep(const Args& a, hipStream_t s) {
  hipLaunchKernelGGL(prep<T>, dim3(a.T, a.G), dim3(256), 2 * a.KP * sizeof(float), s, a);
  return hipGetLastError();
}

template <typename T>
static hipError_t run_scan(const Args& a, hipStream_t s) {
  const dim3 grid((a.V + COLS - 1) / COLS, a.H, a.B);
  switch (a.KP / 32) {
    case 1: hipLaunchKernelGGL((scan<T, 1>), grid, dim3(256), 0, s, a); break;
    case 2: hipLaunchKernelGGL((scan<T, 2>), grid, dim3(256), 0, s, a); break;
    case 3: hipLaunchKernelGGL((scan<T, 3>), grid, dim3(256), 0, s, a); break;
    case 4: hipLaunchKernelGGL((scan<T, 4>), grid, dim3(256), 0, s, a); break;
    case 5: hipLaunchKernelGGL((scan<T, 5>), grid, dim3(256), 0, s, a); break;
    case 6: hipLaunchKernelGGL((scan<T, 6>), grid, dim3(256), 0, s, a); break;
    case 7: hipLaunchKernelGGL((scan<T, 7>), grid, dim3(256), 0, s, a); break;
    case 8: hipLaunchKernelGGL((scan<T, 8>), grid, dim3(256), 0, s, a); break;
    default: return hipErrorInvalidValue;
  }
  return hipGetLastError();
}

}  // namespace delta
}  // namespace kgs

// ptrs: z a2 cw A_log dt_bias row_seq row0 n pos0 slot q k v lg beta qk o S conv (19 device pointers)
// dims: ldz lda oq ok ov ob taps G H K V KP B T f32 (15 values)
KGS_EXPORT int kgs_delta_forward(const void* const* ptrs, const long* dims, hipStream_t s) {
  using namespace kgs::delta;
  Args a{};
  a.z = ptrs[0];
  a.a2 = ptrs[1];
  a.cw = (const float*)ptrs[2];
  a.A_log = (const float*)ptrs[3];
  a.dt_bias = (const float*)ptrs[4];
  a.row_seq = (const int*)ptrs[5];
  a.row0 = (const int*)ptrs[6];
  a.n = (const int*)ptrs[7];
  a.pos0 = (const int*)ptrs[8];
  a.slot = (const int*)ptrs[9];
  a.q = (float*)ptrs[10];
  a.k = (float*)ptrs[11];
  a.v = (float*)ptrs[12];
  a.lg = (float*)ptrs[13];
  a.beta = (float*)ptrs[14];
  a.qk = (float*)ptrs[15];
  a.o = (float*)ptrs[16];
  a.S = (float*)ptrs[17];
  a.conv = (float*)ptrs[18];
  a.ldz = dims[0];
  a.lda = dims[1];
  a.oq = (int)dims[2];
  a.ok = (int)dims[3];
  a.ov = (int)dims[4];
  a.ob = (int)dims[5];
  a.taps = (int)dims[6];
  a.G = (int)dims[7];
  a.H = (int)dims[8];
  a.K = (int)dims[9];
  a.V = (int)dims[10];
  a.KP = (int)dims[11];
  a.B = (int)dims[12];
  a.T = (int)dims[13];
  const bool f32 = dims[14] != 0;
  a.C = 2 * a.G * a.K + a.H * a.V;
  if (a.taps < 1 || a.G < 1 || a.H < 1 || a.H % a.G || a.K < 1 || a.V < 1 || a.B < 1 || a.T < 1 || a.KP % 32 ||
      a.KP < a.K || a.KP > 256 || a.G > 65535 || a.H > 65535 || a.B > 65535)
    return KGS_ERR_SHAPE;
  if (a.ldz < a.oq + a.G * a.K || a.ldz < a.ok + a.G * a.K || a.ldz < a.ov + a.H * a.V || a.ldz < a.ob + a.H ||
      a.lda < (long)a.H * a.K)
    return KGS_ERR_SHAPE;
  hipError_t e = f32 ? run_prep<float>(a, s) : run_prep<unsigned short>(a, s);
  if (e == hipSuccess) e = f32 ? run_scan<float>(a, s) : run_scan<unsigned short>(a, s);
  return (int)e;
}

KGS_EXPORT int kgs_delta_out(const void* o, const void* w, const void* gate, void* y, int T, int H, int V, long ldg,
                             long ldy, float eps, int f32, hipStream_t s) {
  using namespace kgs::delta;
  if (T <= 0 || H <= 0 || V <= 0 || ldg < (long)H * V || ldy < (long)H * V) return KGS_ERR_SHAPE;
  OutArgs a{(const float*)o, (const float*)w, gate, y, ldg, ldy, H, V, eps};
  if (f32) hipLaunchKernelGGL(out<float>, dim3(T), dim3(256), 0, s, a);
  else hipLaunchKernelGGL(out<unsigned short>, dim3(T), dim3(256), 0, s, a);
  return (int)hipGetLastError();
}
