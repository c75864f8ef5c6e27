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
// Short sequences (decode) step token by token:
//   prep   the short causal convolutions + silu of q, k, v (tail of the previous
//          portion from the pool), unit norms, log decays, step sizes;
//   scan   the recurrence.
// Longer ones go by chunks of C = 16 tokens. With b_i the log decays summed from
// the chunk's start, S_0 the state before it and every exponent taken as a
// difference b_i - b_j <= 0 (any decay is safe):
//   A_ij = sum_c k_ic k_jc e^(b_ic - b_jc), P_ij the same with q_i   (j <= i)
//   T = (I + diag(beta) tril(A, -1))^-1 diag(beta)
//   U = T V - (T K~) S_0        K~_i = k_i e^(b_i)
//   O = Q~ S_0 + P U            Q~_i = q_i e^(b_i)
//   S = diag(e^(b_C)) S_0 + K^^T U   K^_j = k_j e^(b_C - b_j)
//   chunk_prep  everything that does not need S_0, one workgroup per (chunk, head);
//   chunk_scan  the three products with the state per chunk, on fp32 MFMAs.
// Both scans also update the convolution tails; out applies the per-head norm and gate.
//
// Everything after the convolutions is fp32. K is padded to KP, a multiple of 32,
// in q, k, log g and the state (pads are zero and stay zero). The state is stored
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
  // the call's two ways: stepped sequences (rows / seqs: their rows and numbers, or
  // null when all are) and chunked ones
  const int *rows, *seqs;
  int nrows, nseqs;
  const int4* chunks;  // per chunk (first row, rows, sequence, -), (sequence's first row, position, slot, -)
  const int4* cseqs;   // (sequence, first chunk, chunks, first row)
  int nchunks, ncseqs;
  float *cW, *cQ, *cK, *cE, *cU, *cP;  // per (chunk, head): [16][KP] x 2, [KP][16], [KP], [16][V], [16][16]
};

// fp32 activations take the precise functions, bf16 ones the hardware's
constexpr float LOG2E = 1.4426950408889634f;
template <bool FAST>
__device__ __forceinline__ float sigm(float x) {
  if constexpr (FAST) return __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-LOG2E * x));
  return 1.0f / (1.0f + expf(-x));
}
// log(1 + e^x); the fast form takes log1p(e) as log(u) e / (u - 1), u = 1 + e, whose
// rounding errors cancel (D. Goldberg, "What Every Computer Scientist Should Know
// About Floating-Point Arithmetic")
template <bool FAST>
__device__ __forceinline__ float softplus(float x) {
  if constexpr (FAST) {
    const float e = __builtin_amdgcn_exp2f(-LOG2E * fabsf(x)), u = 1.0f + e;
    const float l = u == 1.0f ? e : 0.6931471805599453f * __builtin_amdgcn_logf(u) * e * __builtin_amdgcn_rcpf(u - 1.0f);
    return fmaxf(x, 0.f) + l;
  }
  return fmaxf(x, 0.f) + log1pf(expf(-fabsf(x)));
}

// N consecutive channels (1, or 2 on an even boundary)
template <typename T, int N>
__device__ __forceinline__ void ldn(const T* p, float (&v)[N]) {
  if constexpr (N == 2 && sizeof(T) == 2) {
    const unsigned u = *(const unsigned*)p;
    v[0] = bf2f((unsigned short)(u & 0xffff));
    v[1] = bf2f((unsigned short)(u >> 16));
  } else {
#pragma unroll
    for (int i = 0; i < N; ++i) v[i] = ld(p + i);
  }
}

// channels c .. c + N - 1 (column col of z) of row src of the sequence that starts at
// row r0 (position p0): rows ahead of it come from the pool's tail
template <typename T, int N>
__device__ __forceinline__ void conv_in(const Args& a, long src, int c, int col, int r0, int p0, long slot,
                                        float (&x)[N]) {
#pragma unroll
  for (int i = 0; i < N; ++i) x[i] = 0.f;
  if (src >= r0) ldn((const T*)a.z + src * a.ldz + (unsigned)col, x);
  else if (p0 > 0) ldn(a.conv + (slot * (a.taps - 1) + (src - r0 + a.taps - 1)) * a.C + (unsigned)c, x);
}

// ... of row t after the convolution and silu. TAPS 0: any number.
template <typename T, int N, int TAPS>
__device__ __forceinline__ void conv_silu(const Args& a, long t, int c, int col, int r0, int p0, long slot,
                                          float (&y)[N]) {
  float s[N] = {};
  if constexpr (TAPS > 0) {
    float x[TAPS][N];  // all loads are in flight before the first use
#pragma unroll
    for (int j = 0; j < TAPS; ++j) conv_in<T, N>(a, t - (TAPS - 1) + j, c, col, r0, p0, slot, x[j]);
#pragma unroll
    for (int j = 0; j < TAPS; ++j)
#pragma unroll
      for (int i = 0; i < N; ++i) s[i] = __builtin_fmaf(a.cw[(long)j * a.C + c + i], x[j][i], s[i]);
  } else {
    for (int j = 0; j < a.taps; ++j) {
      float x[N];
      conv_in<T, N>(a, t - (a.taps - 1) + j, c, col, r0, p0, slot, x);
#pragma unroll
      for (int i = 0; i < N; ++i) s[i] = __builtin_fmaf(a.cw[(long)j * a.C + c + i], x[i], s[i]);
    }
  }
#pragma unroll
  for (int i = 0; i < N; ++i) y[i] = s[i] * sigm<sizeof(T) == 2>(s[i]);
}

// Rows t0 .. t0 + 15 (n of them real) of channels c .. c + N - 1, each input row read once
template <typename T, int N, int TAPS, class F>
__device__ __forceinline__ void conv_rows(const Args& a, long t0, int n, int c, int col, int r0, int p0, long slot,
                                          F store) {
  if constexpr (TAPS > 0) {
    float x[16 + TAPS - 1][N], w[TAPS][N];
#pragma unroll
    for (int j = 0; j < TAPS; ++j) ldn(a.cw + (long)j * a.C + c, w[j]);
#pragma unroll
    for (int j = 0; j < 16 + TAPS - 1; ++j) {
#pragma unroll
      for (int i = 0; i < N; ++i) x[j][i] = 0.f;
      if (j - (TAPS - 1) < n) conv_in<T, N>(a, t0 - (TAPS - 1) + j, c, col, r0, p0, slot, x[j]);
    }
#pragma unroll
    for (int t = 0; t < 16; ++t) {
      float y[N] = {};
#pragma unroll
      for (int j = 0; j < TAPS; ++j)
#pragma unroll
        for (int i = 0; i < N; ++i) y[i] = __builtin_fmaf(w[j][i], x[t + j][i], y[i]);
#pragma unroll
      for (int i = 0; i < N; ++i) y[i] = t < n ? y[i] * sigm<sizeof(T) == 2>(y[i]) : 0.f;
      store(t, y);
    }
  } else {
    for (int t = 0; t < 16; ++t) {
      float y[N] = {};
      if (t < n) conv_silu<T, N, 0>(a, t0 + t, c, col, r0, p0, slot, y);
      store(t, y);
    }
  }
}

// Where a token's prepared values go
struct Dst {
  float *q, *k, *qk;         // [KP], [KP], one value
  float *v, *lg, *beta;      // of value head h: v + (h - h0) * V, lg + (h - h0) * KP, beta + (h - h0)
};

// One wave: a token's q / k head gh and the value heads h0 .. h0 + nh - 1 that read it
template <typename T, int N, int TAPS>
__device__ __forceinline__ void prep_token(const Args& a, long t, int gh, int h0, int nh, int r0, int p0, long slot,
                                           const Dst& d) {
  constexpr bool FAST = sizeof(T) == 2;
  constexpr int E = 256 / (64 * N);
  const int lane = threadIdx.x & 63, K = a.K, KP = a.KP, V = a.V;
  float q[E][N], k[E][N], sq = 0.f, sk = 0.f, sqk = 0.f;
#pragma unroll
  for (int e = 0; e < E; ++e) {
    const int i = N * (lane + 64 * e);
#pragma unroll
    for (int x = 0; x < N; ++x) q[e][x] = k[e][x] = 0.f;
    if (i < K) {
      const int c = gh * K + i;
      conv_silu<T, N, TAPS>(a, t, c, a.oq + c, r0, p0, slot, q[e]);
      conv_silu<T, N, TAPS>(a, t, a.G * K + c, a.ok + c, r0, p0, slot, k[e]);
#pragma unroll
      for (int x = 0; x < N; ++x) {
        sq = __builtin_fmaf(q[e][x], q[e][x], sq);
        sk = __builtin_fmaf(k[e][x], k[e][x], sk);
        sqk = __builtin_fmaf(q[e][x], k[e][x], sqk);
      }
    }
  }
  sq = wave_sum(sq);
  sk = wave_sum(sk);
  const float rq = 1.0f / sqrtf(sq + 1e-6f) / sqrtf((float)K), rk = 1.0f / sqrtf(sk + 1e-6f);
  sqk = wave_sum(sqk);
  if (lane == 0) *d.qk = sqk * rq * rk;
#pragma unroll
  for (int e = 0; e < E; ++e) {
    const int i = N * (lane + 64 * e);
    if (i < KP) {
#pragma unroll
      for (int x = 0; x < N; ++x) {
        d.q[i + x] = q[e][x] * rq;
        d.k[i + x] = k[e][x] * rk;
      }
    }
  }
  for (int h = h0; h < h0 + nh; ++h) {
    for (int i = N * lane; i < V; i += 64 * N) {
      float v[N];
      const int c = h * V + i;
      conv_silu<T, N, TAPS>(a, t, 2 * a.G * K + c, a.ov + c, r0, p0, slot, v);
#pragma unroll
      for (int x = 0; x < N; ++x) d.v[(h - h0) * V + i + x] = v[x];
    }
    const float A = -expf(a.A_log[h]);
    for (int i = N * lane; i < KP; i += 64 * N) {
      float x[N] = {};
      if (i < K) {
        ldn((const T*)a.a2 + t * a.lda + h * K + i, x);
#pragma unroll
        for (int j = 0; j < N; ++j) x[j] = A * softplus<FAST>(x[j] + a.dt_bias[h * K + i + j]);
      }
#pragma unroll
      for (int j = 0; j < N; ++j) d.lg[(h - h0) * KP + i + j] = x[j];
    }
  }
  if (lane < nh) d.beta[lane] = sigm<FAST>(ld((const T*)a.z + t * a.ldz + a.ob + h0 + lane));
  for (int i = lane + 64; i < nh; i += 64) d.beta[i] = sigm<FAST>(ld((const T*)a.z + t * a.ldz + a.ob + h0 + i));
}

// ----------------------------------------------------------------------- prep
// one wave per (row of a stepped sequence, q / k head)
template <typename T, int N, int TAPS>
__global__ __launch_bounds__(256) void prep(Args a) {
  const long unit = (long)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (unit >= (long)a.nrows * a.G) return;
  const int gh = (int)(unit % a.G), rep = a.H / a.G;
  const long t = a.rows ? a.rows[unit / a.G] : unit / a.G;
  const int b = a.row_seq[t];
  prep_token<T, N, TAPS>(a, t, gh, gh * rep, rep, a.row0[b], a.pos0[b], a.slot[b],
                   Dst{a.q + (t * a.G + gh) * a.KP, a.k + (t * a.G + gh) * a.KP, a.qk + t * a.G + gh,
                       a.v + (t * a.H + gh * rep) * a.V, a.lg + (t * a.H + gh * rep) * a.KP, a.beta + t * a.H + gh * rep});
}

// ----------------------------------------------------------------------- scan
constexpr int TB = 8;     // tokens staged per step
constexpr int COLS = 32;  // state columns per workgroup (4 waves x 8)

__device__ __forceinline__ float xor8_sum(float x) {  // row_ror:8 within 16 lanes
  return x + __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), 0x128, 0xf, 0xf, false));
}

// The convolution tails after the call, the last taps - 1 inputs of the sequence:
// workgroup `part` of `parts` of it takes its share of the channels. Runs in the
// kernel after the one that reads the old tails.
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
  const int b = a.seqs ? a.seqs[blockIdx.z] : blockIdx.z, h = blockIdx.y, c0 = blockIdx.x * COLS;
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

// --------------------------------------------------------------------- chunks
constexpr int CH = 16;  // tokens per chunk

// LDS row pitch: two rows apart are 32 banks apart for n a multiple of 32
__host__ __device__ __forceinline__ int chunk_ld(int n) { return n + 16; }

// 1 / sqrt
template <bool FAST>
__device__ __forceinline__ float rsqrt_(float x) {
  if constexpr (FAST) return __builtin_amdgcn_rsqf(x);
  return 1.0f / sqrtf(x);
}

// one workgroup per (chunk, head). FIX: K = V = FIX, known to the compiler (0: any)
template <typename T, int N, int TAPS, int FIX>
__global__ __launch_bounds__(256, 4) void chunk_prep(Args a) {
  extern __shared__ __attribute__((aligned(16))) float sm[];
  __shared__ __attribute__((aligned(16))) float sA[CH][CH + 4], sT[CH][CH + 4], sbeta[CH], srq[CH], srk[CH];
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6;
  const int K = FIX ? FIX : a.K, KP = FIX ? FIX : a.KP, V = FIX ? FIX : a.V, H = a.H;
  const int ldk = chunk_ld(KP), ldv = chunk_ld(V);
  float *sq = sm, *sk = sq + CH * ldk, *sb = sk + CH * ldk, *sv = sb + CH * ldk;
  const int ck = __builtin_amdgcn_readfirstlane(blockIdx.x / H), h = blockIdx.x - ck * H;
  const int4 it = a.chunks[2 * ck], sq4 = a.chunks[2 * ck + 1];
  const int n = it.y, gh = __builtin_amdgcn_readfirstlane(h / (H / a.G));
  const int r0 = sq4.x, p0 = sq4.y;
  const long slot = sq4.z, t0 = it.x;
  constexpr bool FAST = sizeof(T) == 2;
  // threads by channel groups of N: q, k, v convolutions, then the decays
  const int nk = KP / N, nv = (V + N - 1) / N;
  for (int u = tid; u < 3 * nk + nv; u += 256) {
    if (u < 2 * nk) {
      const bool isk = u >= nk;
      const int c = N * (isk ? u - nk : u);
      float* dst = (isk ? sk : sq) + c;
      auto put = [&](int t, const float (&y)[N]) {
#pragma unroll
        for (int i = 0; i < N; ++i) dst[t * ldk + i] = y[i];
      };
      const int ch = (isk ? a.G * K : 0) + gh * K + c, col = (isk ? a.ok : a.oq) + gh * K + c;
      if (c < K) conv_rows<T, N, TAPS>(a, t0, n, ch, col, r0, p0, slot, put);
      else
        for (int t = 0; t < CH; ++t) put(t, {});
    } else if (u < 2 * nk + nv) {
      const int c = N * (u - 2 * nk);
      conv_rows<T, N, TAPS>(a, t0, n, 2 * a.G * K + h * V + c, a.ov + h * V + c, r0, p0, slot,
                            [&](int t, const float (&y)[N]) {
#pragma unroll
                              for (int i = 0; i < N; ++i) sv[t * ldv + c + i] = y[i];
                            });
    } else {
      const int c = N * (u - 2 * nk - nv);
      const float A = -expf(a.A_log[h]) * LOG2E;  // b: sums of log decays, in log2 units
      float s[N] = {}, dt[N] = {};
      if (c < K) ldn(a.dt_bias + h * K + c, dt);
      float x[CH][N];
#pragma unroll
      for (int t = 0; t < CH; ++t) {
#pragma unroll
        for (int i = 0; i < N; ++i) x[t][i] = 0.f;
        if (t < n && c < K) ldn((const T*)a.a2 + (t0 + t) * a.lda + h * K + (unsigned)c, x[t]);
      }
#pragma unroll
      for (int t = 0; t < CH; ++t)
#pragma unroll
        for (int i = 0; i < N; ++i) {
          if (t < n && c < K) s[i] += A * softplus<FAST>(x[t][i] + dt[i]);
          sb[t * ldk + c + i] = s[i];
        }
    }
  }
  if (tid < CH) sbeta[tid] = tid < n ? sigm<FAST>(ld((const T*)a.z + (t0 + tid) * a.ldz + a.ob + h)) : 0.f;
  __syncthreads();
  for (int i = w; i < CH; i += 4) {  // unit norms, as factors
    float ssq = 0.f, ssk = 0.f, sqk = 0.f;
    for (int c = lane; c < KP; c += 64) {
      const float q = sq[i * ldk + c], k = sk[i * ldk + c];
      ssq = __builtin_fmaf(q, q, ssq);
      ssk = __builtin_fmaf(k, k, ssk);
      sqk = __builtin_fmaf(q, k, sqk);
    }
    ssq = wave_sum(ssq);
    ssk = wave_sum(ssk);
    sqk = wave_sum(sqk);
    if (lane == 0) {
      const float rq = rsqrt_<FAST>(ssq + 1e-6f) * rsqrt_<FAST>((float)K), rk = rsqrt_<FAST>(ssk + 1e-6f);
      srq[i] = rq;
      srk[i] = rk;
      a.cP[((long)ck * H + h) * CH * CH + i * CH + i] = sqk * rq * rk;  // P's diagonal has no decay
    }
  }
  __syncthreads();
  const long base = (long)ck * H + h;
  float* P = a.cP + base * CH * CH;
  // A and P in 2 x 2 tiles of (i, j): 28 tiles below the diagonal over 8 slices of the
  // channels each, and the 8 pairs (2 x + 1, 2 x) on it over 4 slices
  if (tid < 224) {
    const int blk = tid >> 3, sl = tid & 7;
    int bi = 1;
    while ((bi + 1) * bi / 2 <= blk) ++bi;
    const int i = 2 * bi, j = 2 * (blk - bi * (bi - 1) / 2);
    float sa[2][2] = {}, sp[2][2] = {};
    for (int c = 4 * sl; c < KP; c += 32) {
      f32x4 ki[2], qi[2], xi[2], kj[2], xj[2];
#pragma unroll
      for (int y = 0; y < 2; ++y) {
        ki[y] = *(const f32x4*)(sk + (i + y) * ldk + c);
        qi[y] = *(const f32x4*)(sq + (i + y) * ldk + c);
        xi[y] = *(const f32x4*)(sb + (i + y) * ldk + c);
        kj[y] = *(const f32x4*)(sk + (j + y) * ldk + c);
        xj[y] = *(const f32x4*)(sb + (j + y) * ldk + c);
      }
#pragma unroll
      for (int y = 0; y < 2; ++y)
#pragma unroll
        for (int z = 0; z < 2; ++z)
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            const float v = kj[z][e] * __builtin_amdgcn_exp2f(xi[y][e] - xj[z][e]);
            sa[y][z] = __builtin_fmaf(ki[y][e], v, sa[y][z]);
            sp[y][z] = __builtin_fmaf(qi[y][e], v, sp[y][z]);
          }
    }
#pragma unroll
    for (int y = 0; y < 2; ++y)
#pragma unroll
      for (int z = 0; z < 2; ++z) {
        const float ra = sum8(sa[y][z]), rp = sum8(sp[y][z]);
        if (sl == 2 * y + z) {
          const float f = srk[j + z];
          sA[i + y][j + z] = ra * srk[i + y] * f;
          P[(i + y) * CH + j + z] = rp * srq[i + y] * f;
          P[(j + z) * CH + i + y] = 0.f;
        }
      }
  } else {
    const int j = 2 * ((tid - 224) >> 2), i = j + 1, sl = tid & 3;
    float sa = 0.f, sp = 0.f;
    for (int c = 4 * sl; c < KP; c += 16) {
      const f32x4 ki = *(const f32x4*)(sk + i * ldk + c), qi = *(const f32x4*)(sq + i * ldk + c);
      const f32x4 xi = *(const f32x4*)(sb + i * ldk + c), kj = *(const f32x4*)(sk + j * ldk + c);
      const f32x4 xj = *(const f32x4*)(sb + j * ldk + c);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const float v = kj[e] * __builtin_amdgcn_exp2f(xi[e] - xj[e]);
        sa = __builtin_fmaf(ki[e], v, sa);
        sp = __builtin_fmaf(qi[e], v, sp);
      }
    }
    sa += dpp_move<0xB1>(sa);
    sp += dpp_move<0xB1>(sp);
    sa += dpp_move<0x4E>(sa);
    sp += dpp_move<0x4E>(sp);
    if (sl == 0) {
      sA[i][j] = sa * srk[i] * srk[j];
      P[i * CH + j] = sp * srq[i] * srk[j];
      P[j * CH + i] = 0.f;
    }
  }
  __syncthreads();
  if (tid < CH) {  // column tid of T by forward substitution
    float t[CH];
#pragma unroll
    for (int i = 0; i < CH; ++i) {
      asm volatile("" ::: "memory");
      float s = 0.f;
#pragma unroll
      for (int m = 0; m < i; ++m) s = __builtin_fmaf(sA[i][m], t[m], s);
      t[i] = i < tid ? 0.f : i == tid ? sbeta[i] : -sbeta[i] * s;
      sT[i][tid] = t[i];
    }
  }
  __syncthreads();
  // T K~, Q~, K^^T and e^(b_C) per key channel, T V per value channel
  for (int c = tid; c < KP + V; c += 256) {
    float x[CH];
    if (c < KP) {
      float *Q = a.cQ + base * CH * KP, *Kt = a.cK + base * KP * CH;
      const float bc = sb[(CH - 1) * ldk + c];
#pragma unroll
      for (int i = 0; i < CH; ++i) {
        const float bi = sb[i * ldk + c], k = sk[i * ldk + c] * srk[i], e = __builtin_amdgcn_exp2f(bi);
        x[i] = k * e;
        Q[(unsigned)(i * KP + c)] = sq[i * ldk + c] * srq[i] * e;
      }
#pragma unroll
      for (int i = 0; i < CH; i += 4) {
        f32x4 v;
#pragma unroll
        for (int y = 0; y < 4; ++y)
          v[y] = sk[(i + y) * ldk + c] * srk[i + y] * __builtin_amdgcn_exp2f(bc - sb[(i + y) * ldk + c]);
        *(f32x4*)(Kt + (unsigned)(c * CH + i)) = v;
      }
      a.cE[base * KP + c] = __builtin_amdgcn_exp2f(bc);
    } else {
#pragma unroll
      for (int i = 0; i < CH; ++i) x[i] = sv[i * ldv + c - KP];
    }
    float* W = a.cW + base * CH * KP;
    float* U = a.cU + base * CH * V;
#pragma unroll
    for (int i = 0; i < CH; ++i) {
      asm volatile("" ::: "memory");  // T's rows are read here, not all kept in registers
      float s = 0.f;
#pragma unroll
      for (int j = 0; j <= i; j += 4) {
        const f32x4 t = *(const f32x4*)&sT[i][j];  // zero above the diagonal
#pragma unroll
        for (int y = 0; y < 4; ++y) s = __builtin_fmaf(t[y], x[j + y], s);
      }
      if (c < KP) W[(unsigned)(i * KP + c)] = s;
      else U[(unsigned)(i * V + c - KP)] = s;
    }
  }
}

// One workgroup per (sequence, head, 16 NS state columns); wave w holds the state's
// 16-row tiles w, w + 4, ... as MFMA accumulators: lane (g = lane >> 4, n = lane & 15)
// has rows 4 g + r of a tile for columns n, 16 + n, .... Register r of an accumulator
// is at the same time the B operand of a v_mfma_f32_16x16x4_f32 whose four
// contraction indices are 4 g + r, so state and U feed the products without
// moving; the A operands are read as float4s in that order. The waves' partial
// products over their rows meet in LDS, one barrier per chunk.
// NS 2 reads the A operands half as often; NS 1 spreads few heads over more CUs.
template <typename T, int MT, int NS>
__global__ __launch_bounds__(256) void chunk_scan(Args a) {
  __shared__ f32x4 part[2][2][NS][4][64];  // [buffer][U | O][tile][wave][lane]
  const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int l16 = lane & 15, g = lane >> 4;
  const int KP = a.KP, V = a.V, H = a.H, nslab = (V + 16 * NS - 1) / (16 * NS), ntile = KP / 16;
  const int lid = xcd_remap(blockIdx.x, gridDim.x);  // a head's slabs share an XCD's L2
  // (divisions run on the vector unit: back to scalars, so that bases stay uniform)
  const int sh = __builtin_amdgcn_readfirstlane(lid / nslab), slab = __builtin_amdgcn_readfirstlane(lid - sh * nslab);
  const int si = __builtin_amdgcn_readfirstlane(sh / H), h = sh - si * H;
  const int4 sq = a.cseqs[si];  // sequence, first chunk, chunks, first row
  const int b = sq.x, n = a.n[b];
  int col[NS];
  bool live[NS];
  f32x4 S[MT][NS];
  float* Sh = a.S + ((long)a.slot[b] * H + h) * V * KP + 4 * g;
#pragma unroll
  for (int s = 0; s < NS; ++s) {
    col[s] = (slab * NS + s) * 16 + l16;
    live[s] = col[s] < V;
    col[s] = min(col[s], V - 1);
#pragma unroll
    for (int m = 0; m < MT; ++m) {
      const int tile = w + 4 * m;
      S[m][s] = tile < ntile && a.pos0[b] > 0 ? *(const f32x4*)(Sh + (long)col[s] * KP + 16 * tile) : f32x4{};
    }
  }
  struct Frag {
    f32x4 W[MT], Q[MT], K[MT], E[MT], U[NS], P;
  };
  // Loads without conditions (a wave's rows past the last tile repeat it, columns
  // past V the last one), so that the number in flight is known at every wait;
  // a uniform base and 32-bit lane offsets.
  unsigned lw[MT], lk[MT], le[MT], lu[NS];
#pragma unroll
  for (int m = 0; m < MT; ++m) {
    const int tile = min(w + 4 * m, ntile - 1);
    lw[m] = l16 * KP + 16 * tile + 4 * g;
    lk[m] = (16 * tile + l16) * CH + 4 * g;
    le[m] = 16 * tile + 4 * g;
  }
#pragma unroll
  for (int s = 0; s < NS; ++s) lu[s] = 4 * g * V + col[s];
  const unsigned lp = l16 * CH + 4 * g;
  auto fetch = [&](int c, Frag& f) {
    const long base = (long)(sq.y + c) * H + h;
    const float *W = a.cW + base * CH * KP, *Q = a.cQ + base * CH * KP, *K = a.cK + base * CH * KP;
    const float *E = a.cE + base * KP, *U = a.cU + base * CH * V, *P = a.cP + base * CH * CH;
#pragma unroll
    for (int m = 0; m < MT; ++m) {
      f.W[m] = *(const f32x4*)(W + lw[m]);
      f.Q[m] = *(const f32x4*)(Q + lw[m]);
      f.K[m] = *(const f32x4*)(K + lk[m]);
      f.E[m] = *(const f32x4*)(E + le[m]);
    }
#pragma unroll
    for (int s = 0; s < NS; ++s)
#pragma unroll
      for (int r = 0; r < 4; ++r) f.U[s][r] = (U + (unsigned)(r * V))[lu[s]];
    f.P = *(const f32x4*)(P + lp);
    __builtin_amdgcn_sched_barrier(0);  // chunks are loaded in order: their waits are counted in it
  };
  // a ring of RING chunks' operands in registers: loads run RING - 1 chunks ahead
  constexpr int RING = MT == 1 || (MT == 2 && NS == 1) ? 4 : MT == 2 ? 3 : 2;
  auto step = [&](int c, Frag& f) __attribute__((always_inline)) {
    f32x4 pu[NS], po[NS];
#pragma unroll
    for (int s = 0; s < NS; ++s) pu[s] = po[s] = f32x4{};
#pragma unroll
    for (int m = 0; m < MT; ++m)
#pragma unroll
      for (int r = 0; r < 4; ++r)
#pragma unroll
        for (int s = 0; s < NS; ++s) {
          pu[s] = __builtin_amdgcn_mfma_f32_16x16x4f32(f.W[m][r], S[m][s][r], pu[s], 0, 0, 0);
          po[s] = __builtin_amdgcn_mfma_f32_16x16x4f32(f.Q[m][r], S[m][s][r], po[s], 0, 0, 0);
        }
    const int buf = c & 1;
#pragma unroll
    for (int s = 0; s < NS; ++s) {
      part[buf][0][s][w][lane] = pu[s];
      part[buf][1][s][w][lane] = po[s];
    }
    __syncthreads();
    f32x4 U[NS];
#pragma unroll
    for (int s = 0; s < NS; ++s)
      U[s] = f.U[s] - (part[buf][0][s][0][lane] + part[buf][0][s][1][lane] + part[buf][0][s][2][lane] +
                       part[buf][0][s][3][lane]);
#pragma unroll
    for (int m = 0; m < MT; ++m)
#pragma unroll
      for (int s = 0; s < NS; ++s) S[m][s] *= f.E[m];
#pragma unroll
    for (int r = 0; r < 4; ++r)
#pragma unroll
      for (int m = 0; m < MT; ++m)
#pragma unroll
        for (int s = 0; s < NS; ++s)
          S[m][s] = __builtin_amdgcn_mfma_f32_16x16x4f32(f.K[m][r], U[s][r], S[m][s], 0, 0, 0);
#pragma unroll
    for (int m = 0; m < MT; ++m)
      if (w + 4 * m >= ntile) {  // no such rows
#pragma unroll
        for (int s = 0; s < NS; ++s) S[m][s] = f32x4{};
      }
#pragma unroll
    for (int s = 0; s < NS; ++s)
      if (w == ((c + 2 * s) & 3)) {
        f32x4 O = part[buf][1][s][0][lane] + part[buf][1][s][1][lane] + part[buf][1][s][2][lane] +
                  part[buf][1][s][3][lane];
#pragma unroll
        for (int r = 0; r < 4; ++r) O = __builtin_amdgcn_mfma_f32_16x16x4f32(f.P[r], U[s][r], O, 0, 0, 0);
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int t = CH * c + 4 * g + r;
          if (t < n && live[s]) a.o[((long)(sq.w + t) * H + h) * V + col[s]] = O[r];
        }
      }
    fetch(min(c + RING, sq.z - 1), f);
  };
  Frag f0, f1, f2, f3;
  fetch(0, f0);
  fetch(min(1, sq.z - 1), f1);
  if constexpr (RING > 2) fetch(min(2, sq.z - 1), f2);
  if constexpr (RING > 3) fetch(min(3, sq.z - 1), f3);
  int c = 0;
  for (; c + RING <= sq.z; c += RING) {
    step(c, f0);
    step(c + 1, f1);
    if constexpr (RING > 2) step(c + 2, f2);
    if constexpr (RING > 3) step(c + 3, f3);
  }
  if (c < sq.z) step(c, f0);
  if constexpr (RING > 2)
    if (c + 1 < sq.z) step(c + 1, f1);
  if constexpr (RING > 3)
    if (c + 2 < sq.z) step(c + 2, f2);
#pragma unroll
  for (int s = 0; s < NS; ++s)
    if (live[s]) {
#pragma unroll
      for (int m = 0; m < MT; ++m)
        if (w + 4 * m < ntile) *(f32x4*)(Sh + (long)col[s] * KP + 16 * (w + 4 * m)) = S[m][s];
    }
  conv_tail<T>(a, b, h * nslab + slab, H * nslab);
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

// one wave per (row, head)
template <typename T>
__global__ __launch_bounds__(256) void out(OutArgs a) {
  constexpr bool FAST = sizeof(T) == 2;
  const int lane = threadIdx.x & 63, V = a.V;
  const long t = blockIdx.x;
  const int h = blockIdx.y * 4 + (threadIdx.x >> 6);
  T* y = (T*)a.y + t * a.ldy;
  if (blockIdx.y == 0)
    for (int i = a.H * V + threadIdx.x; i < a.ldy; i += 256) st(y + i, 0.f);
  if (h >= a.H) return;
  const T* gate = (const T*)a.gate + t * a.ldg + h * V;
  const float* o = a.o + (t * a.H + h) * V;
  y += h * V;
  if (V == 128) {
    const float2 x = *(const float2*)(o + 2 * lane);
    float gt[2];
    ldn<T, 2>(gate + 2 * lane, gt);
    const float2 w = *(const float2*)(a.w + 2 * lane);
    const float r = 1.0f / sqrtf(wave_sum(x.x * x.x + x.y * x.y) / V + a.eps);
    const float y0 = x.x * r * w.x * sigm<FAST>(gt[0]), y1 = x.y * r * w.y * sigm<FAST>(gt[1]);
    if constexpr (FAST) *(unsigned*)(y + 2 * lane) = pack_bf16x2(y0, y1);
    else *(float2*)(y + 2 * lane) = make_float2(y0, y1);
    return;
  }
  float ss = 0.f;
  for (int i = lane; i < V; i += 64) ss += o[i] * o[i];
  const float r = 1.0f / sqrtf(wave_sum(ss) / V + a.eps);
  for (int i = lane; i < V; i += 64) st(y + i, o[i] * r * a.w[i] * sigm<FAST>(ld(gate + i)));
}

template <typename T, int NS>
static void run_chunk_scan(const Args& a, hipStream_t s) {
  const dim3 grid((unsigned)((a.V + 16 * NS - 1) / (16 * NS) * a.H * a.ncseqs));
  switch ((a.KP + 63) / 64) {
    case 1: hipLaunchKernelGGL((chunk_scan<T, 1, NS>), grid, dim3(256), 0, s, a); break;
    case 2: hipLaunchKernelGGL((chunk_scan<T, 2, NS>), grid, dim3(256), 0, s, a); break;
    case 3: hipLaunchKernelGGL((chunk_scan<T, 3, NS>), grid, dim3(256), 0, s, a); break;
    default: hipLaunchKernelGGL((chunk_scan<T, 4, NS>), grid, dim3(256), 0, s, a); break;
  }
}

template <typename T, int N, int TAPS>
static hipError_t run(const Args& a, hipStream_t s) {
  if (a.nrows > 0) {
    const long units = (long)a.nrows * a.G;
    hipLaunchKernelGGL((prep<T, N, TAPS>), dim3((unsigned)((units + 3) / 4)), dim3(256), 0, s, a);
    const dim3 grid((a.V + COLS - 1) / COLS, a.H, a.nseqs);
    switch (a.KP / 32) {
      case 1: hipLaunchKernelGGL((scan<T, 1>), grid, dim3(256), 0, s, a); break;
      case 2: hipLaunchKernelGGL((scan<T, 2>), grid, dim3(256), 0, s, a); break;
      case 3: hipLaunchKernelGGL((scan<T, 3>), grid, dim3(256), 0, s, a); break;
      case 4: hipLaunchKernelGGL((scan<T, 4>), grid, dim3(256), 0, s, a); break;
      case 5: hipLaunchKernelGGL((scan<T, 5>), grid, dim3(256), 0, s, a); break;
      case 6: hipLaunchKernelGGL((scan<T, 6>), grid, dim3(256), 0, s, a); break;
      case 7: hipLaunchKernelGGL((scan<T, 7>), grid, dim3(256), 0, s, a); break;
      default: hipLaunchKernelGGL((scan<T, 8>), grid, dim3(256), 0, s, a); break;
    }
  }
  if (a.nchunks > 0) {
    const size_t lds = sizeof(float) * CH * (3 * chunk_ld(a.KP) + chunk_ld(a.V));
    auto prep_k = chunk_prep<T, N, TAPS, 0>;
    if constexpr (N == 2 && TAPS == 4)
      if (a.K == 128 && a.KP == 128 && a.V == 128) prep_k = chunk_prep<T, N, TAPS, 128>;
    if (lds > 48 * 1024) {
      const hipError_t e =
          hipFuncSetAttribute((const void*)prep_k, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
      if (e != hipSuccess) return e;
    }
    hipLaunchKernelGGL(prep_k, dim3((unsigned)(a.nchunks * a.H)), dim3(256), lds, s, a);
    const long wide = (long)((a.V + 31) / 32) * a.H * a.ncseqs;
    if (a.V > 16 && wide >= 256) run_chunk_scan<T, 2>(a, s);
    else run_chunk_scan<T, 1>(a, s);
  }
  return hipGetLastError();
}

template <typename T>
static hipError_t run(const Args& a, bool pairs, hipStream_t s) {
  if (pairs) return a.taps == 4 ? run<T, 2, 4>(a, s) : run<T, 2, 0>(a, s);
  return run<T, 1, 0>(a, s);
}

}  // namespace delta
}  // namespace kgs

// ptrs (29 device pointers): z a2 cw A_log dt_bias row_seq row0 n pos0 slot q k v lg beta qk o S conv
//   rows seqs chunks cseqs cW cQ cK cE cU cP
// dims (20): ldz lda oq ok ov ob taps G H K V KP B T f32 nrows nseqs nchunks ncseqs, even (channel pairs aligned)
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
  a.rows = (const int*)ptrs[19];
  a.seqs = (const int*)ptrs[20];
  a.chunks = (const int4*)ptrs[21];
  a.cseqs = (const int4*)ptrs[22];
  a.cW = (float*)ptrs[23];
  a.cQ = (float*)ptrs[24];
  a.cK = (float*)ptrs[25];
  a.cE = (float*)ptrs[26];
  a.cU = (float*)ptrs[27];
  a.cP = (float*)ptrs[28];
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
  const bool f32 = dims[14] != 0, pairs = dims[19] != 0;
  a.nrows = (int)dims[15];
  a.nseqs = (int)dims[16];
  a.nchunks = (int)dims[17];
  a.ncseqs = (int)dims[18];
  a.C = 2 * a.G * a.K + a.H * a.V;
  if (a.taps < 1 || a.G < 1 || a.H < 1 || a.H % a.G || a.K < 1 || a.V < 1 || a.B < 1 || a.T < 1 || a.KP % 32 ||
      a.KP < a.K || a.KP > 256 || a.G > 65535 || a.H > 65535 || a.B > 65535)
    return KGS_ERR_SHAPE;
  if (a.ldz < a.oq + a.G * a.K || a.ldz < a.ok + a.G * a.K || a.ldz < a.ov + a.H * a.V || a.ldz < a.ob + a.H ||
      a.lda < (long)a.H * a.K)
    return KGS_ERR_SHAPE;
  if (a.nrows < 0 || a.nseqs < 0 || a.nchunks < 0 || a.ncseqs < 0 || a.nseqs > 65535 || a.V > 1024 ||
      (a.nrows > 0) != (a.nseqs > 0) || (a.nchunks > 0) != (a.ncseqs > 0) || (long)a.nchunks * a.H > 0x7fffffff)
    return KGS_ERR_SHAPE;
  if (a.nchunks > 0 && (!a.chunks || !a.cseqs || !a.cW || !a.cQ || !a.cK || !a.cE || !a.cU || !a.cP)) return KGS_ERR_ARG;
  if (pairs && (a.K % 2 || a.V % 2 || (a.ldz | a.lda | a.oq | a.ok | a.ov) % 2 || ((uintptr_t)a.z | (uintptr_t)a.a2) & 3))
    return KGS_ERR_ALIGN;
  return (int)(f32 ? run<float>(a, pairs, s) : run<unsigned short>(a, pairs, s));
}

KGS_EXPORT int kgs_delta_out(const void* o, const void* w, const void* gate, void* y, int T, int H, int V, long ldg,
                             long ldy, float eps, int f32, hipStream_t s) {
  using namespace kgs::delta;
  if (T <= 0 || H <= 0 || V <= 0 || ldg < (long)H * V || ldy < (long)H * V) return KGS_ERR_SHAPE;
  OutArgs a{(const float*)o, (const float*)w, gate, y, ldg, ldy, H, V, eps};
  if (V == 128 && (ldg % 2 || ldy % 2 || ((uintptr_t)gate & 3) || (((uintptr_t)o | (uintptr_t)w | (uintptr_t)y) & 7)))
    return KGS_ERR_ALIGN;
  const dim3 grid(T, (H + 3) / 4);
  if (f32) hipLaunchKernelGGL(out<float>, grid, dim3(256), 0, s, a);
  else hipLaunchKernelGGL(out<unsigned short>, grid, dim3(256), 0, s, a);
  return (int)hipGetLastError();
}
