// Linear attention with one fixed decay per head (lightning attention) for gfx950: per
// sequence and head a K x V state S in fp32, for each token
//
//   S <- d S + k v^T;  o = S^T q        q, k, v = silu of the projections
//
// Sequences of a call are ragged: sequence b is rows row0[b] .. row0[b] + n[b] - 1 at
// positions pos0[b] .., its state in slot[b] of the pool; pos0 = 0 starts from zeros
// whatever the slot holds, so freeing a slot needs no clear.
//
//   step    token by token, the state in registers: decode, short portions, fp32.
//   chunks  longer portions in bf16, C = 64 tokens at a time, every power of the decay
//           from a table (any decay is safe). With S_0 the state before the chunk:
//             O^T = d^(i+1) S_0^T Q^T + V^T P^T,  P_ij = d^(i-j) q_i . k_j  (j <= i)
//             S   = d^n S_0 + K^T V',             V'_j = d^(n-1-j) v_j
//           q, k and v are bf16 MFMA operands; P, V' and S enter the products as two bf16
//           parts each (16 bits) and S itself stays in the fp32 accumulators: a wave owns
//           16 columns of V, and the accumulator layout of S is the operand layout of
//           S^T for keys in the order Q is staged in.
//           A long portion is cut into segments that run side by side: chunks without
//           output give every segment's own contribution, `scan` turns them into the
//           states the segments start from.
//   out     RMS norm over all heads together, weight, sigmoid gate.
//
// K is padded to KP, V to VP with zero columns in the projections (silu(0) = 0 keeps the
// state's padding zero). State: [slot][head][KP][VP].
#include <type_traits>

#include "kgs_common.h"

namespace kgs {
namespace lightning {

constexpr int C = 64;    // tokens of a chunk
constexpr int PLD = 72;  // row of P in LDS

struct Args {
  const void* z;       // [T, ldz]: q, k, v from columns oq, ok, ov, head by head
  long ldz;
  int oq, ok, ov;
  const int* row0;     // [B]
  const int* n;
  const int* pos0;
  const int* slot;
  const int* seqs;     // step: the sequences that step, or null: all
  const int4* items;   // chunks: (sequence, first token of the segment, tokens, its buffer or -1)
  const int4* scans;   // scan: (sequence, first buffer, segments, chunks of a full segment)
  const float* dec;    // [H][C + 1] powers of the decay
  const float* decc;   // [H][nc + 1] powers of d^C
  float* S;            // [slots][H][KP][VP]
  float* buf;          // [buffers][H][KP][VP]
  float* o;            // [T][H VP]
  int H, KP, VP, nc;
};

// N consecutive elements, aligned to 4 of them
template <int N>
__device__ __forceinline__ void ldn(const float* p, float (&v)[N]) {
#pragma unroll
  for (int i = 0; i < N; i += 4) {
    const f32x4 x = *(const f32x4*)(p + i);
#pragma unroll
    for (int j = 0; j < 4; ++j) v[i + j] = x[j];
  }
}
template <int N>
__device__ __forceinline__ void ldn(const unsigned short* p, float (&v)[N]) {
  constexpr int W = N % 8 ? 4 : 8;
  typedef short vec __attribute__((ext_vector_type(W)));
#pragma unroll
  for (int i = 0; i < N; i += W) {
    const vec x = *(const vec*)(p + i);
#pragma unroll
    for (int j = 0; j < W; ++j) v[i + j] = bf2f((unsigned short)x[j]);
  }
}
// precise where everything is fp32
template <bool FAST>
__device__ __forceinline__ float silu(float z) {
  if constexpr (FAST) return z * __builtin_amdgcn_rcpf(1.0f + __expf(-z));
  return z / (1.0f + expf(-z));
}

// ------------------------------------------------------------------------ step
// Eight row groups of KR keys x 32 lanes of 4 columns; grid: V slab of 128, head, sequence
template <typename T, int KR>
__global__ __launch_bounds__(256) void step(Args a) {
  constexpr bool FAST = sizeof(T) == 2;
  constexpr int KP = 8 * KR;
  __shared__ __attribute__((aligned(16))) float red[2][8][128];
  const int b = a.seqs ? a.seqs[blockIdx.z] : blockIdx.z, h = blockIdx.y, rg = threadIdx.x >> 5, cx = threadIdx.x & 31;
  const int col = blockIdx.x * 128 + 4 * cx;
  const bool live = col < a.VP;
  const int n = a.n[b];
  const long row0 = a.row0[b];
  const float d = a.dec[h * (C + 1) + 1];
  float* Sp = a.S + (((long)a.slot[b] * a.H + h) * KP + rg * KR) * a.VP + col;
  const T* z = (const T*)a.z + row0 * a.ldz;
  const T* qp = z + a.oq + h * KP + rg * KR;
  const T* kp = z + a.ok + h * KP + rg * KR;
  const T* vp = z + a.ov + h * a.VP + col;
  f32x4 S[KR];
  const bool fresh = a.pos0[b] == 0;
#pragma unroll
  for (int i = 0; i < KR; ++i) S[i] = live && !fresh ? *(const f32x4*)(Sp + (long)i * a.VP) : f32x4{};
  for (int t = 0; t < n; ++t) {
    const long zo = t * a.ldz;
    float v[4] = {}, kz[KR], qz[KR];
    if (live) ldn(vp + zo, v);
    ldn(kp + zo, kz);
    ldn(qp + zo, qz);
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = silu<FAST>(v[i]);
    f32x4 o{};
#pragma unroll
    for (int i = 0; i < KR; ++i) {
      const float k = silu<FAST>(kz[i]), q = silu<FAST>(qz[i]);
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        S[i][j] = __builtin_fmaf(k, v[j], d * S[i][j]);
        o[j] = __builtin_fmaf(q, S[i][j], o[j]);
      }
    }
    *(f32x4*)(&red[t & 1][rg][4 * cx]) = o;
    __syncthreads();  // also: the readers of two tokens ago are done
    if (rg == 0 && live) {
#pragma unroll
      for (int g = 1; g < 8; ++g) o += *(const f32x4*)(&red[t & 1][g][4 * cx]);
      *(f32x4*)(a.o + ((row0 + t) * a.H + h) * a.VP + col) = o;
    }
  }
  if (live)
#pragma unroll
    for (int i = 0; i < KR; ++i) *(f32x4*)(Sp + (long)i * a.VP) = S[i];
}

// ---------------------------------------------------------------------- chunks
typedef unsigned u32x4 __attribute__((ext_vector_type(4)));

// two bf16 parts of eight fp32 values
__device__ __forceinline__ void split8(const float (&x)[8], bf16x8& hi, bf16x8& lo) {
  u32x4 h, l;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    h[i] = pack_bf16x2(x[2 * i], x[2 * i + 1]);
    l[i] = pack_bf16x2(x[2 * i] - __uint_as_float(h[i] << 16), x[2 * i + 1] - __uint_as_float(h[i] & 0xffff0000u));
  }
  hi = __builtin_bit_cast(bf16x8, h);
  lo = __builtin_bit_cast(bf16x8, l);
}

__device__ __forceinline__ bf16x8 silu8(bf16x8 x) {
  float y[8];
#pragma unroll
  for (int i = 0; i < 8; ++i) y[i] = silu<true>(bf2f((unsigned short)x[i]));
  return pack_bf16x8(y, 0);
}

// grid: (item, head, V slab of 16 NW); NK: 32-key blocks; a wave has 16 columns of V. OUT: with output, from the
// segment's starting state; else the segment's own contribution into its buffer.
template <int NK, int NW, bool OUT>
__global__ __launch_bounds__(64 * NW, 4) void chunks(Args a) {
  constexpr int KP = 32 * NK, QLD = KP + 8, VS = 16 * NW, VLD = VS + 8, NT = 64 * NW;
  constexpr int UK = C * KP / 8 / NT, UV = C * VS / 8 / NT;  // 16-B units per thread
  __shared__ __attribute__((aligned(16))) unsigned short Qs[OUT ? C * QLD : 8];
  __shared__ __attribute__((aligned(16))) unsigned short Ks[C * QLD];
  __shared__ __attribute__((aligned(16))) unsigned short Vs[C * VLD];
  __shared__ __attribute__((aligned(16))) unsigned short Ps[2][OUT ? C * PLD : 8];  // rows i, columns j; hi, lo
  __shared__ float dec[C + 1];
  int tid = threadIdx.x, n = tid & 15, q = tid >> 4 & 3;
  const int w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int nslab = a.VP / VS;
  int id = blockIdx.x;
  const int slab = id % nslab;
  id /= nslab;
  const int h = id % a.H;
  const int4 it = a.items[id / a.H];
  if (!OUT && it.w < 0) return;
  const long row0 = a.row0[it.x] + it.y;
  const bool last = it.y + it.z == a.n[it.x];
  if (!OUT && last) return;  // nothing starts from its end
  for (int i = tid; i <= C; i += NT) dec[i] = a.dec[h * (C + 1) + i];

  const long per = (long)KP * a.VP;
  float* pool = a.S + ((long)a.slot[it.x] * a.H + h) * per;
  const int vcol = slab * VS + 16 * w + n;
  f32x4 S[2 * NK];
  bool live = false;  // the state is not zero
  {
    const float* src = nullptr;
    if (OUT) src = it.w >= 0 ? a.buf + ((long)it.w * a.H + h) * per : a.pos0[it.x] > 0 ? pool : nullptr;
    live = src != nullptr;
#pragma unroll
    for (int kt = 0; kt < 2 * NK; ++kt)
#pragma unroll
      for (int r = 0; r < 4; ++r) S[kt][r] = live ? src[(long)(16 * kt + 4 * q + r) * a.VP + vcol] : 0.f;
  }

  const unsigned short* z = (const unsigned short*)a.z + row0 * a.ldz;
  const unsigned short* zq = z + a.oq + h * KP;
  const unsigned short* zk = z + a.ok + h * KP;
  const unsigned short* zv = z + a.ov + h * a.VP + slab * VS;
  bf16x8 rq[OUT ? UK : 1], rk[UK], rv[UV];
  const unsigned ld = a.ldz;  // a segment's rows are within 32-bit offsets
  auto fetch = [&](int c0) {  // a chunk's projections, rows past the end zero
    const int nr = it.z - c0;
#pragma unroll
    for (int i = 0; i < UK; ++i) {
      const int u = tid + i * NT, r = u / (KP / 8), c = u % (KP / 8);
      const unsigned o = (unsigned)(c0 + r) * ld + 8 * c;
      if constexpr (OUT) rq[i] = r < nr ? *(const bf16x8*)(zq + o) : bf16x8{};
      rk[i] = r < nr ? *(const bf16x8*)(zk + o) : bf16x8{};
    }
#pragma unroll
    for (int i = 0; i < UV; ++i) {
      const int u = tid + i * NT, r = u / (VS / 8), c = u % (VS / 8);
      rv[i] = r < nr ? *(const bf16x8*)(zv + (unsigned)(c0 + r) * ld + 8 * c) : bf16x8{};
    }
  };
  // 8 tokens (32 ks + 8 q ..) of column col + n of a row-major tile
  auto column = [&](const unsigned short* t, int ldt, int ks, int col) {
    const unsigned short* p = t + (32 * ks + 8 * q + (n >> 2)) * ldt + col + 4 * (n & 3);
    return tr_frag((const char*)p, (const char*)(p + 4 * ldt));
  };

  fetch(0);
  for (int c0 = 0; c0 < it.z; c0 += C) {
    const int nc = min(C, it.z - c0);
    // addresses are worked out anew for every chunk: kept over the loop they would not fit the registers
    asm volatile("" : "+v"(tid), "+v"(n), "+v"(q));
#pragma unroll
    for (int i = 0; i < UK; ++i) {
      const int u = tid + i * NT, r = u / (KP / 8), c = u % (KP / 8);
      *(bf16x8*)(Ks + r * QLD + 8 * c) = silu8(rk[i]);
      if constexpr (OUT) {
        // keys of a 32-block in the order 0-3, 16-19, 4-7, 20-23, ..
        const bf16x8 x = silu8(rq[i]);
        const int g = 2 * (c & 3);
        unsigned short* p = Qs + r * QLD + 32 * (c >> 2);
        *(bf16x4*)(p + 8 * (g & 3) + 4 * (g >> 2)) = __builtin_shufflevector(x, x, 0, 1, 2, 3);
        *(bf16x4*)(p + 8 * ((g + 1) & 3) + 4 * ((g + 1) >> 2)) = __builtin_shufflevector(x, x, 4, 5, 6, 7);
      }
    }
#pragma unroll
    for (int i = 0; i < UV; ++i) {
      const int u = tid + i * NT, r = u / (VS / 8), c = u % (VS / 8);
      *(bf16x8*)(Vs + r * VLD + 8 * c) = silu8(rv[i]);
    }
    __syncthreads();
    if (!OUT && c0 + C < it.z) fetch(c0 + C);

    bf16x8 vf[2];
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) vf[ks] = column(Vs, VLD, ks, 16 * w);

    if constexpr (OUT) {
      // tiles of P: P^T, a lane has 4 neighbouring j of one i; a wave has one row of tiles or half of it
      {
        constexpr int NS = NW / 4;
        const int ti = w & 3, i = 16 * ti + n;
        bf16x8 qf[NK];
#pragma unroll
        for (int t = 0; t < NK; ++t) qf[t] = *(const bf16x8*)(Qs + i * QLD + 32 * t + 8 * q);
        for (int tj = w >> 2; tj <= (ti | 1); tj += NS) {
          f32x4 p{};
          if (tj <= ti) {
#pragma unroll
            for (int t = 0; t < NK; ++t) {
              const unsigned short* kp = Ks + (16 * tj + n) * QLD + 32 * t + 4 * q;
              const bf16x4 x = *(const bf16x4*)kp, y = *(const bf16x4*)(kp + 16);
              p = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_shufflevector(x, y, 0, 1, 2, 3, 4, 5, 6, 7), qf[t], p, 0,
                                                          0, 0);
            }
          }
          uint2 hi, lo;
          float v[4];
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            const int j = 16 * tj + 4 * q + r;
            v[r] = j <= i ? p[r] * dec[max(i - j, 0)] : 0.f;
          }
          hi = make_uint2(pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3]));
          lo = make_uint2(pack_bf16x2(v[0] - __uint_as_float(hi.x << 16), v[1] - __uint_as_float(hi.x & 0xffff0000u)),
                          pack_bf16x2(v[2] - __uint_as_float(hi.y << 16), v[3] - __uint_as_float(hi.y & 0xffff0000u)));
          *(uint2*)(Ps[0] + i * PLD + 16 * tj + 4 * q) = hi;
          *(uint2*)(Ps[1] + i * PLD + 16 * tj + 4 * q) = lo;
        }
      }
      f32x4 acc[4];
#pragma unroll
      for (int ti = 0; ti < 4; ++ti) acc[ti] = f32x4{};
      if (live) {
#pragma unroll
        for (int t = 0; t < NK; ++t) {
          __builtin_amdgcn_sched_barrier(0);
          bf16x8 sh, sl, qf[4];
#pragma unroll
          for (int ti = 0; ti < 4; ++ti) qf[ti] = *(const bf16x8*)(Qs + (16 * ti + n) * QLD + 32 * t + 8 * q);
          float x[8];
#pragma unroll
          for (int e = 0; e < 4; ++e) x[e] = S[2 * t][e], x[4 + e] = S[2 * t + 1][e];
          split8(x, sh, sl);
#pragma unroll
          for (int ti = 0; ti < 4; ++ti) acc[ti] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(sl, qf[ti], acc[ti], 0, 0, 0);
#pragma unroll
          for (int ti = 0; ti < 4; ++ti) acc[ti] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(sh, qf[ti], acc[ti], 0, 0, 0);
        }
#pragma unroll
        for (int ti = 0; ti < 4; ++ti) acc[ti] *= dec[16 * ti + n + 1];
      }
      __syncthreads();  // P is there
      if (c0 + C < it.z) fetch(c0 + C);  // in flight from here on, where fewer registers are needed
      __builtin_amdgcn_sched_barrier(0);
#pragma unroll
      for (int ti = 0; ti < 4; ++ti)
#pragma unroll
        for (int ks = 0; ks <= ti / 2; ++ks) {
          const unsigned short* pp = Ps[0] + (16 * ti + n) * PLD + 32 * ks + 8 * q;
          const bf16x8 ph = *(const bf16x8*)pp, pl = *(const bf16x8*)(pp + (Ps[1] - Ps[0]));
          acc[ti] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[ks], pl, acc[ti], 0, 0, 0);
          acc[ti] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[ks], ph, acc[ti], 0, 0, 0);
        }
#pragma unroll
      for (int ti = 0; ti < 4; ++ti) {
        const int i = 16 * ti + n;
        if (i >= nc) continue;
        *(f32x4*)(a.o + ((row0 + c0 + i) * a.H + h) * a.VP + slab * VS + 16 * w + 4 * q) = acc[ti];
      }
    }

    // the state after the chunk
    {
      const float dn = dec[nc];
#pragma unroll
      for (int kt = 0; kt < 2 * NK; ++kt) S[kt] *= dn;
    }
#pragma unroll
    for (int ks = 0; ks < 2; ++ks) {
      bf16x8 vh, vl;
      float x[8];
#pragma unroll
      for (int e = 0; e < 8; ++e)  // rows past the end are zero
        x[e] = dec[max(nc - 1 - (32 * ks + 8 * q + e), 0)] * bf2f((unsigned short)vf[ks][e]);
      split8(x, vh, vl);
#pragma unroll
      for (int kt = 0; kt < 2 * NK; ++kt) {
        const bf16x8 kf = column(Ks, QLD, ks, 16 * kt);
        S[kt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, vl, S[kt], 0, 0, 0);
        S[kt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, vh, S[kt], 0, 0, 0);
      }
    }
    live = true;
    __syncthreads();  // the chunk in LDS is used
  }
  if (OUT && !last) return;
  float* dst = OUT ? pool : a.buf + ((long)it.w * a.H + h) * per;
#pragma unroll
  for (int kt = 0; kt < 2 * NK; ++kt)
#pragma unroll
    for (int r = 0; r < 4; ++r) dst[(long)(16 * kt + 4 * q + r) * a.VP + vcol] = S[kt][r];
}

// the segments' contributions -> the states they start from; grid: 1024 floats of a state, head, sequence
__global__ __launch_bounds__(256) void scan(Args a) {
  const int h = blockIdx.y;
  const int4 sc = a.scans[blockIdx.z];
  const long per = (long)a.KP * a.VP, i = ((long)blockIdx.x * 256 + threadIdx.x) * 4;
  if (i >= per) return;
  const float d = a.decc[h * (a.nc + 1) + sc.w];
  f32x4 S{};
  if (a.pos0[sc.x] > 0) S = *(const f32x4*)(a.S + ((long)a.slot[sc.x] * a.H + h) * per + i);
  float* p = a.buf + ((long)sc.y * a.H + h) * per + i;
  const long st = a.H * per;
  constexpr int U = 4;
  for (int s = 0; s < sc.z; s += U) {
    f32x4 x[U];
#pragma unroll
    for (int u = 0; u < U; ++u) x[u] = s + u + 1 < sc.z ? *(const f32x4*)(p + (s + u) * st) : f32x4{};
#pragma unroll
    for (int u = 0; u < U; ++u)
      if (s + u < sc.z) {
        *(f32x4*)(p + (s + u) * st) = S;
        S = d * S + x[u];
      }
  }
}

// ------------------------------------------------------------------------- out
struct OutArgs {
  const float* o;    // [T, n]
  const float* w;    // [n]
  const void* gate;  // [T, ldg]
  void* y;           // [T, ldy], columns n .. ldy zeroed
  long ldg, ldy;
  int n, count;      // columns, and those that are not padding
  float eps;
};

// one workgroup per row, NV groups of 4 columns per thread
template <typename T, int NV>
__global__ __launch_bounds__(256) void out(OutArgs a) {
  constexpr bool FAST = sizeof(T) == 2;
  __shared__ float part[4];
  const long t = blockIdx.x;
  const int tid = threadIdx.x, nt = blockDim.x;
  const T* g = (const T*)a.gate + t * a.ldg;
  T* y = (T*)a.y + t * a.ldy;
  f32x4 x[NV], gt[NV];
  float ss = 0.f;
#pragma unroll
  for (int k = 0; k < NV; ++k) {
    const int c = 4 * (tid + k * nt);
    x[k] = c < a.n ? *(const f32x4*)(a.o + t * a.n + c) : f32x4{};
    float e[4] = {};
    if (c < a.n) ldn(g + c, e);
#pragma unroll
    for (int i = 0; i < 4; ++i) gt[k][i] = e[i];
#pragma unroll
    for (int i = 0; i < 4; ++i) ss = __builtin_fmaf(x[k][i], x[k][i], ss);
  }
  ss = wave_sum(ss);
  if (nt > 64) {
    if ((tid & 63) == 0) part[tid >> 6] = ss;
    __syncthreads();
    ss = part[0];
    for (int i = 1; i < nt / 64; ++i) ss += part[i];
  }
  const float inv = 1.0f / sqrtf(ss / a.count + a.eps);
#pragma unroll
  for (int k = 0; k < NV; ++k) {
    const int c = 4 * (tid + k * nt);
    if (c >= a.n) continue;
    const f32x4 w = *(const f32x4*)(a.w + c);
    float v[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const float e = FAST ? __expf(-gt[k][i]) : expf(-gt[k][i]);
      v[i] = x[k][i] * inv * w[i] / (1.0f + e);
    }
    if constexpr (FAST) *(uint2*)(y + c) = make_uint2(pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3]));
    else *(f32x4*)(y + c) = f32x4{v[0], v[1], v[2], v[3]};
  }
  for (int c = a.n + 4 * tid; c < a.ldy; c += 4 * nt) {
    if constexpr (FAST) *(uint2*)(y + c) = make_uint2(0, 0);
    else *(f32x4*)(y + c) = f32x4{};
  }
}

template <typename T>
void run_step(const Args& a, int nseqs, hipStream_t s) {
  const dim3 grid((a.VP + 127) / 128, a.H, nseqs);
  if (a.KP == 64) hipLaunchKernelGGL((step<T, 8>), grid, dim3(256), 0, s, a);
  else if (a.KP == 128) hipLaunchKernelGGL((step<T, 16>), grid, dim3(256), 0, s, a);
  else hipLaunchKernelGGL((step<T, 32>), grid, dim3(256), 0, s, a);
}

template <bool OUT>
void run_chunks(const Args& a, int nitems, hipStream_t s) {
  const int nw = a.VP == 64 ? 4 : 8;
  const dim3 grid((unsigned)((long)nitems * a.H * (a.VP / (16 * nw)))), block(64 * nw);
  if (a.KP == 64) {
    if (nw == 4) hipLaunchKernelGGL((chunks<2, 4, OUT>), grid, block, 0, s, a);
    else hipLaunchKernelGGL((chunks<2, 8, OUT>), grid, block, 0, s, a);
  } else {
    if (nw == 4) hipLaunchKernelGGL((chunks<4, 4, OUT>), grid, block, 0, s, a);
    else hipLaunchKernelGGL((chunks<4, 8, OUT>), grid, block, 0, s, a);
  }
}

template <typename T>
int run_out(const OutArgs& a, int rows, hipStream_t s) {
  const int nc = a.n / 4, nt = nc >= 256 ? 256 : (nc + 63) / 64 * 64, nv = (nc + nt - 1) / nt;
  const dim3 grid(rows), block(nt);
  if (nv <= 1) hipLaunchKernelGGL((out<T, 1>), grid, block, 0, s, a);
  else if (nv <= 2) hipLaunchKernelGGL((out<T, 2>), grid, block, 0, s, a);
  else if (nv <= 4) hipLaunchKernelGGL((out<T, 4>), grid, block, 0, s, a);
  else if (nv <= 8) hipLaunchKernelGGL((out<T, 8>), grid, block, 0, s, a);
  else hipLaunchKernelGGL((out<T, 16>), grid, block, 0, s, a);
  return (int)hipGetLastError();
}

}  // namespace lightning
}  // namespace kgs

// z [T, ldz] holds q, k, v from columns oq, ok, ov, H heads of KP (64, 128, 256) and VP (64
// or a multiple of 128) columns, padding zero. nstep sequences (seqs, or all of them) go
// token by token; nitems segments (bf16, KP <= 128) by chunks of 64: (sequence, first token,
// tokens, buffer or -1), nscan sequences of several segments (sequence, first buffer,
// segments, chunks of a full segment <= nc), whose segments' buffers follow one another.
// dec [H][65]: d^0 .. d^64, decc [H][nc + 1]: powers of d^64. o fp32 [T][H VP].
KGS_EXPORT int kgs_lightning_forward(const void* z, long ldz, int oq, int ok, int ov, const void* row0, const void* n,
                                     const void* pos0, const void* slot, const void* seqs, int nstep, const void* items,
                                     int nitems, const void* scans, int nscan, const void* dec, const void* decc, int nc,
                                     void* S, void* buf, void* o, int H, int KP, int VP, int f32, hipStream_t s) {
  using namespace kgs::lightning;
  if (H <= 0 || H > 65535 || (KP != 64 && KP != 128 && KP != 256) || VP <= 0 || (VP != 64 && VP % 128) || nstep < 0 ||
      nstep > 65535 || nitems < 0 || nscan < 0 || nscan > 65535 || nc < 0 || ldz < oq + H * KP || ldz < ok + H * KP ||
      ldz < ov + H * VP || (long)nitems * H * (VP / 64) > 0x7fffffff)
    return KGS_ERR_SHAPE;
  if (nitems > 0 && (f32 || KP > 128 || !items)) return KGS_ERR_ARG;
  if (nscan > 0 && (!scans || !buf || !nitems)) return KGS_ERR_ARG;
  if (ldz % 8 || oq % 8 || ok % 8 || ov % 8 ||
      (((uintptr_t)z | (uintptr_t)S | (uintptr_t)buf | (uintptr_t)o | (uintptr_t)items | (uintptr_t)scans) & 15))
    return KGS_ERR_ALIGN;
  Args a{z, ldz, oq, ok, ov, (const int*)row0, (const int*)n, (const int*)pos0, (const int*)slot, (const int*)seqs,
         (const int4*)items, (const int4*)scans, (const float*)dec, (const float*)decc, (float*)S, (float*)buf, (float*)o,
         H, KP, VP, nc};
  if (nstep > 0) {
    if (f32) run_step<float>(a, nstep, s);
    else run_step<unsigned short>(a, nstep, s);
  }
  if (nitems > 0) {
    if (nscan > 0) {
      run_chunks<false>(a, nitems, s);
      hipLaunchKernelGGL(scan, dim3((KP * VP / 4 + 255) / 256, H, nscan), dim3(256), 0, s, a);
    }
    run_chunks<true>(a, nitems, s);
  }
  return (int)hipGetLastError();
}

// y = norm(o row of n columns, `count` of them real) * w * sigmoid(gate)
KGS_EXPORT int kgs_lightning_out(const void* o, const void* w, const void* gate, long ldg, void* y, long ldy, int T, int n,
                                 int count, float eps, int f32, hipStream_t s) {
  using namespace kgs::lightning;
  if (T <= 0 || n <= 0 || n % 4 || n > 16384 || count <= 0 || count > n || ldg < n || ldy < n || ldy % 4) return KGS_ERR_SHAPE;
  if (ldg % 4 || (((uintptr_t)o | (uintptr_t)w | (uintptr_t)y | (uintptr_t)gate) & 15)) return KGS_ERR_ALIGN;
  OutArgs a{(const float*)o, (const float*)w, gate, y, ldg, ldy, n, count, eps};
  return f32 ? run_out<float>(a, T, s) : run_out<unsigned short>(a, T, s);
}
