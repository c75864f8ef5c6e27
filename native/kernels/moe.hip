// Mixture-of-experts feed-forward for gfx950.
//
//   route    router logits (bf16: MFMA with fp32 sums; fp32: plain dot products), the
//            `top` largest per token and their sigmoid weights, and each choice's rank
//            among the tokens of its expert (counted in LDS per 16 tokens, one global
//            add per expert and workgroup). The other choice: softmax scores, chosen by
//            score + correction within the best groups of neighbours, weights normalised;
//            outputs past the experts return the input (their weights' sum is put out)
//            and one more router row can be a shared expert's gate
//   plan     a prefix over the experts' counts turns ranks into rows of the sorted
//            order: row -> token and weight, choice -> row, and the GEMM tiles
//            (expert, first row, rows)
//   grouped  the experts' GEMMs over that order on the four-wave K-loop of gemm_w4.h:
//            gate|up reads its A rows straight from the tokens' activations by LDS-DMA
//            with per-lane row offsets and applies weight, clamps and gate in the
//            epilogue; down reads the sorted rows. Neither reads anything back on the
//            host: the grid covers the most tiles there can be and the rest leaves.
//
// A weight scales its expert's input or its output. Both projections of an expert are
// linear in the input, so there it multiplies their fp32 sums, before the clamps; down is
// linear too, so a weight of the output multiplies the gated product in fp32.
#include "gemm_w4.h"
#include "kgs_common.h"

namespace kgs {
namespace moe {

constexpr int RT = 16;  // tokens per route workgroup

struct RouteArgs {
  const void* h;      // [T, ldh]
  long ldh;
  const void* w;      // [ep, wp], expert rows padded to a multiple of 16
  const int* slots;   // [T] or null: rows with slot < 0 are padding and choose nothing
  int* counts;        // [E], zero
  int* ids;           // [T, top]
  int* rank;          // [T, top]
  float* weight;      // [T, top]
  int T, E, ep, wp, top;
  // softmax scores: E experts and `extra` outputs that return the input
  const float* corr;  // [E + extra], or null: sigmoid scores, nothing below is used
  float* ident;       // [T] sum of the weights of the extra outputs a token chose, or null
  float* gate;        // [T] sigmoid of router row E + extra, or null
  int extra, groups, keep;
  float scale;
};

__device__ __forceinline__ float rcp_sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }

// the larger logit, the lower number on a tie, over the 16 lanes of a DPP row
template <int CTRL>
__device__ __forceinline__ void better(float& v, int& e) {
  const float ov = dpp_move<CTRL>(v);
  const int oe = __float_as_int(dpp_move<CTRL>(__int_as_float(e)));
  if (ov > v || (ov == v && oe < e)) v = ov, e = oe;
}

// z[16 tokens][zs] in LDS -> choices; 16 lanes per token (the first 256 threads), each over
// its own experts
__device__ __forceinline__ void choose(const RouteArgs& a, float* z, int zs, int* lh, int t0) {
  const int tid = threadIdx.x, tk = tid >> 4, n = tid & 15, nt = blockDim.x;
  for (int e = tid; e < a.E; e += nt) lh[e] = 0;
  __syncthreads();
  const int t = t0 + tk;
  const bool real = tid < 256 && t < a.T && (!a.slots || a.slots[t] >= 0);
  if (tid < 256) {
    float* row = z + tk * zs;
    for (int k = 0; k < a.top; ++k) {
      float best = -INFINITY;
      int be = 0x7fffffff;
      for (int e = n; e < a.E; e += 16) {
        const float v = row[e];
        if (v > best || (be == 0x7fffffff && v == best)) best = v, be = e;
      }
      better<0x128>(best, be);  // row_ror 8, 4, 2, 1
      better<0x124>(best, be);
      better<0x122>(best, be);
      better<0x121>(best, be);
      // be is a valid expert unless every logit left is NaN: such a token takes none
      const bool ok = be < a.E;
      if (ok && (be & 15) == n) row[be] = __uint_as_float(0x7fc00000u);  // taken: compares false from now on
      if (n == 0 && t < a.T) {
        const long o = (long)t * a.top + k;
        a.ids[o] = real && ok ? be : -1;
        a.weight[o] = rcp_sigmoid(best);
        a.rank[o] = real && ok ? atomicAdd(&lh[be], 1) : 0;
      }
    }
  }
  __syncthreads();
  // local ranks -> ranks among all tokens
  for (int e = tid; e < a.E; e += nt) {
    const int c = lh[e];
    if (c) lh[e] = atomicAdd(&a.counts[e], c);
  }
  __syncthreads();
  if (n == 0 && real)
    for (int k = 0; k < a.top; ++k) {
      const long o = (long)t * a.top + k;
      if (a.ids[o] >= 0) a.rank[o] += lh[a.ids[o]];
    }
}

__device__ __forceinline__ float row_max(float v) {  // over the 16 lanes of a DPP row
  v = fmaxf(v, dpp_move<0x128>(v));
  v = fmaxf(v, dpp_move<0x124>(v));
  v = fmaxf(v, dpp_move<0x122>(v));
  return fmaxf(v, dpp_move<0x121>(v));
}
__device__ __forceinline__ float row_sum(float v) {
  v += dpp_move<0x128>(v);
  v += dpp_move<0x124>(v);
  v += dpp_move<0x122>(v);
  return v + dpp_move<0x121>(v);
}

// The same for softmax scores (p: [16][zs], scratch): work [16][groups + 2 top] after the E counters
__device__ __forceinline__ void choose_softmax(const RouteArgs& a, float* z, float* p, int zs, int* lh, int t0) {
  const int tid = threadIdx.x, tk = tid >> 4, n = tid & 15, nt = blockDim.x, EA = a.E + a.extra;
  float* best_of = (float*)(lh + a.E);           // [16][groups]
  float* lw = best_of + RT * a.groups;           // [16][top]
  int* lid = (int*)(lw + RT * a.top);            // [16][top]
  for (int e = tid; e < a.E; e += nt) lh[e] = 0;
  __syncthreads();
  const int t = t0 + tk, per = EA / a.groups;
  const bool on = tid < 256, real = on && t < a.T && (!a.slots || a.slots[t] >= 0);
  float* row = z + tk * zs;
  float* pr = p + tk * zs;
  if (on) {
    float m = -INFINITY, s = 0.f;
    for (int e = n; e < EA; e += 16) m = fmaxf(m, row[e]);
    m = row_max(m);
    for (int e = n; e < EA; e += 16) s += pr[e] = expf(row[e] - m);
    s = row_sum(s);
    for (int e = n; e < EA; e += 16) {
      pr[e] /= s;
      row[e] = pr[e] + a.corr[e];  // choice score
    }
  }
  __syncthreads();
  if (a.keep < a.groups) {
    if (on)
      for (int g = n; g < a.groups; g += 16) {
        float b = row[g * per];
        for (int i = 1; i < per; ++i) b = fmaxf(b, row[g * per + i]);
        best_of[tk * a.groups + g] = b;
      }
    __syncthreads();
    if (on)
      for (int g = n; g < a.groups; g += 16) {
        const float b = best_of[tk * a.groups + g];
        int ahead = 0;
        for (int j = 0; j < a.groups; ++j) {
          const float o = best_of[tk * a.groups + j];
          ahead += o > b || (o == b && j < g);
        }
        if (ahead >= a.keep)
          for (int i = 0; i < per; ++i) row[g * per + i] = __uint_as_float(0x7fc00000u);  // compares false
      }
    __syncthreads();
  }
  if (on) {
    float sum = 0.f;
    for (int k = 0; k < a.top; ++k) {
      float best = -INFINITY;
      int be = 0x7fffffff;
      for (int e = n; e < EA; e += 16) {
        const float v = row[e];
        if (v > best || (be == 0x7fffffff && v == best)) best = v, be = e;
      }
      better<0x128>(best, be);
      better<0x124>(best, be);
      better<0x122>(best, be);
      better<0x121>(best, be);
      const bool ok = be < EA;
      const float s = ok ? pr[be] : 0.f;
      if (ok && (be & 15) == n) row[be] = __uint_as_float(0x7fc00000u);
      sum += s;
      if (n == 0) {
        lid[tk * a.top + k] = ok ? be : -1;
        lw[tk * a.top + k] = s;
      }
    }
    if (n == 0) best_of[tk * a.groups] = a.scale / (sum + 1e-20f);
  }
  __syncthreads();
  for (int i = tid; i < RT * a.top; i += nt) {
    const int k = i / a.top, tt = t0 + k;
    if (tt >= a.T) continue;
    const int e = lid[i];
    const bool ok = e >= 0 && e < a.E && (!a.slots || a.slots[tt] >= 0);
    const long o = (long)tt * a.top + (i - k * a.top);
    a.ids[o] = ok ? e : -1;
    a.weight[o] = lw[i] * best_of[k * a.groups];
    a.rank[o] = ok ? atomicAdd(&lh[e], 1) : 0;
  }
  if (on && n == 0 && t < a.T) {
    if (a.ident) {
      float w = 0.f;
      for (int k = 0; k < a.top; ++k)
        if (lid[tk * a.top + k] >= a.E) w += lw[tk * a.top + k];
      a.ident[t] = real ? w * best_of[tk * a.groups] : 0.f;
    }
    if (a.gate) a.gate[t] = rcp_sigmoid(row[EA]);
  }
  __syncthreads();
  for (int e = tid; e < a.E; e += nt) {  // local ranks -> ranks among all tokens
    const int c = lh[e];
    if (c) lh[e] = atomicAdd(&a.counts[e], c);
  }
  __syncthreads();
  for (int i = tid; i < RT * a.top; i += nt) {  // the thread that wrote it
    const int k = i / a.top, tt = t0 + k;
    if (tt >= a.T) continue;
    const long o = (long)tt * a.top + (i - k * a.top);
    const int e = a.ids[o];
    if (e >= 0) a.rank[o] += lh[e];
  }
}

// bf16: eight waves split the width, ET 16-expert MFMA tiles each, U steps' loads at a time
template <int ET>
__global__ __launch_bounds__(512) void route_mfma(RouteArgs a) {
  constexpr int U = ET >= 4 ? 2 : 8;
  extern __shared__ float lds[];
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, n = lane & 15, q = lane >> 4;
  const int t0 = blockIdx.x * RT, t = min(t0 + n, a.T - 1), kw = a.wp / 8;
  const unsigned short* hp = (const unsigned short*)a.h + (long)t * a.ldh + w * kw + 8 * q;
  const unsigned short* wr = (const unsigned short*)a.w + (long)n * a.wp + w * kw + 8 * q;
  f32x4 acc[ET];
#pragma unroll
  for (int e = 0; e < ET; ++e) acc[e] = f32x4{};
  auto steps = [&](int k, auto uc) {
    constexpr int UU = decltype(uc)::value;
    bf16x8 hf[UU], wf[UU][ET];
#pragma unroll
    for (int u = 0; u < UU; ++u) {
      hf[u] = *(const bf16x8*)(hp + k + 32 * u);
#pragma unroll
      for (int e = 0; e < ET; ++e) wf[u][e] = *(const bf16x8*)(wr + (long)e * 16 * a.wp + k + 32 * u);
    }
#pragma unroll
    for (int u = 0; u < UU; ++u)
#pragma unroll
      for (int e = 0; e < ET; ++e) acc[e] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[u][e], hf[u], acc[e], 0, 0, 0);
  };
  int k = 0;
  for (; k + 32 * U <= kw; k += 32 * U) steps(k, std::integral_constant<int, U>{});
  for (; k < kw; k += 32) steps(k, std::integral_constant<int, 1>{});
  // lane: token n, experts 16e + 4q + r; the waves' sums meet in LDS, added in wave order
  const int zs = a.ep + 1;
  float* z = lds;
  float* part = lds + RT * zs;  // [8][RT][zs]
  int* lh = (int*)(part + 8 * RT * zs);
#pragma unroll
  for (int e = 0; e < ET; ++e)
#pragma unroll
    for (int r = 0; r < 4; ++r) part[(w * RT + n) * zs + 16 * e + 4 * q + r] = acc[e][r];
  __syncthreads();
  for (int i = threadIdx.x; i < RT * zs; i += 512) {
    float s = part[i];
#pragma unroll
    for (int j = 1; j < 8; ++j) s += part[j * RT * zs + i];
    z[i] = s;
  }
  // both begin with a barrier
  if (a.corr) choose_softmax(a, z, part, zs, lh, t0);
  else choose(a, z, zs, lh, t0);
}

template <typename T>
__global__ __launch_bounds__(256) void route_plain(RouteArgs a) {
  extern __shared__ float lds[];
  const int zs = a.ep + 1, t0 = blockIdx.x * RT, tk = threadIdx.x >> 4, n = threadIdx.x & 15;
  float* z = lds;
  float* p = lds + RT * zs;
  int* lh = (int*)(a.corr ? p + RT * zs : p);
  const int nrow = a.E + a.extra + (a.gate ? 1 : 0);
  const T* hp = (const T*)a.h + (long)min(t0 + tk, a.T - 1) * a.ldh;
  for (int e = 0; e < nrow; ++e) {
    const T* wr = (const T*)a.w + (long)e * a.wp;
    float s = 0.f;
    for (int k = n; k < a.wp; k += 16) {
      if constexpr (sizeof(T) == 2) s = __builtin_fmaf(bf2f(hp[k]), bf2f(wr[k]), s);
      else s = __builtin_fmaf(hp[k], wr[k], s);
    }
#pragma unroll
    for (int x = 1; x < 16; x <<= 1) s += __shfl_xor(s, x, 16);
    if (n == 0) z[tk * zs + e] = s;
  }
  __syncthreads();
  if (a.corr) choose_softmax(a, z, p, zs, lh, t0);
  else choose(a, z, zs, lh, t0);
}

struct PlanArgs {
  const int* counts;
  const int* ids;
  const int* rank;
  const float* weight;
  int* pos;       // [T, top] sorted row of each choice, -1: none
  int* rows;      // [T * top] token of each sorted row
  float* roww;    // [T * top] its weight
  int4* tiles;    // (expert, first row, rows, 0)
  int* ntiles;
  int n, top, E, bm;
};

__global__ __launch_bounds__(1024) void plan(PlanArgs a) {
  __shared__ int off[1024], til[1024];
  const int tid = threadIdx.x;
  const int c = tid < a.E ? a.counts[tid] : 0, nt = (c + a.bm - 1) / a.bm;
  off[tid] = c;
  til[tid] = nt;
  __syncthreads();
  for (int d = 1; d < a.E; d <<= 1) {  // inclusive prefix
    const int o = tid >= d ? off[tid - d] : 0, u = tid >= d ? til[tid - d] : 0;
    __syncthreads();
    off[tid] += o;
    til[tid] += u;
    __syncthreads();
  }
  if (blockIdx.x == 0) {
    const int r0 = off[tid] - c, i0 = til[tid] - nt;
    for (int i = 0; i < nt; ++i) a.tiles[i0 + i] = make_int4(tid, r0 + i * a.bm, min(a.bm, c - i * a.bm), 0);
    if (tid == a.E - 1) *a.ntiles = til[tid];
  }
  const int i = blockIdx.x * 1024 + tid;
  if (i >= a.n) return;
  const int e = a.ids[i];
  if (e < 0) {
    a.pos[i] = -1;
    return;
  }
  const int p = (e ? off[e - 1] : 0) + a.rank[i];
  a.pos[i] = p;
  a.rows[p] = i / a.top;
  a.roww[p] = a.weight[i];
}

struct GroupedArgs {
  const void* A;       // gate|up: tokens' activations [T, lda]; down: sorted rows
  const void* B;       // [E][N][K]
  void* C;             // [P, ldc] (SPLIT: fp32 [slice][P][N])
  const int* rows;
  const float* roww;
  const int4* tiles;
  const int* ntiles;
  long lda;
  int T, P, N, K, ldc, nslice;
  float limit;
  int act;             // ACT_*
};

// the clamped gate of a weighted input; silu(gate) up, the product weighted
enum { ACT_CLAMPED = 0, ACT_SILU = 1 };
__device__ __forceinline__ float gated_weighted(float g, float u, float w, const GroupedArgs& a) {
  if (a.act == ACT_SILU) return gate_act<GATE_SILU>(g) * u * w;
  return gate_clamped(g * w, u * w, a.limit);
}

// GATED: gate|up with gathered rows and the gated epilogue; else the down projection,
// SPLIT over K into fp32 partial products or whole in bf16.
template <int BM, int BN, int NS, bool GATED, bool SPLIT>
__global__ __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(1, 1))) void grouped(GroupedArgs a) {
  using namespace w4;
  using S = Shape<BM, BN>;
  constexpr int MA = S::MA, NB = S::NB, ND = dma_per_stage<BM, BN>();
  constexpr int X = GATED ? 3000000 : 0;
  using KN = Knobs<BM, BN>;
  static_assert(NS * S::STAGE <= 160 * 1024, "LDS stages exceed 160 KiB");
  __shared__ __attribute__((aligned(1024))) char smem[NS * S::STAGE];
  const int ntm = *a.ntiles, ntn = a.N / BN;
  if ((int)blockIdx.x >= ntm * ntn * (SPLIT ? a.nslice : 1)) return;
  const int lane = threadIdx.x & 63;
  const int w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  int slice, tm, tn;
  tile_of<X % 100, SPLIT>((int)blockIdx.x, ntm * ntn * (SPLIT ? a.nslice : 1), ntm, ntn, slice, tm, tn);
  const int4 tile = a.tiles[tm];
  const int row0 = tile.y, nrow = tile.z, lda = (int)a.lda, ldb = a.K * (SPLIT ? a.nslice : 1);
  const long koff = (long)slice * a.K;
  const unsigned short* A = (const unsigned short*)a.A;
  const unsigned short* B = (const unsigned short*)a.B + (long)tile.x * a.N * ldb;

  Ctx c;
  c.smem = smem;
  c.w = w;
  c.wr = w >> 1;
  c.wc = w & 1;
  c.nt = a.K / BK;
  if constexpr (GATED) {
    c.ra = __builtin_amdgcn_make_buffer_rsrc((void*)A, 0, (int)(a.T * a.lda * 2), 0x00020000);
    c.rb = __builtin_amdgcn_make_buffer_rsrc((void*)(B + (long)tn * (BN / 2) * ldb), 0, (BN / 2) * ldb * 2, 0x00020000);
    c.rb2 = __builtin_amdgcn_make_buffer_rsrc((void*)(B + ((long)a.N / 2 + (long)tn * (BN / 2)) * ldb), 0,
                                              (BN / 2) * ldb * 2, 0x00020000);
  } else {
    c.ra = __builtin_amdgcn_make_buffer_rsrc((void*)(A + (long)row0 * lda + koff), 0, (nrow * lda - (int)koff) * 2, 0x00020000);
    c.rb = __builtin_amdgcn_make_buffer_rsrc((void*)(B + (long)tn * BN * ldb + koff), 0, (BN * ldb - (int)koff) * 2, 0x00020000);
  }
  c.sa32 = 32 * lda * 2;
  c.sb32 = 32 * ldb * 2;
  {
    const int row = w * 8 + (lane >> 3);
    const int ch = (lane & 7) ^ ((row >> 1) & 7);
    c.voa = (row * lda + ch * 8) * 2;
    c.vob = (row * ldb + ch * 8) * 2;
    if constexpr (GATED) {
#pragma unroll
      for (int j = 0; j < BM / 32; ++j)
        c.vog[j] = (int)(((long)a.rows[row0 + min(j * 32 + row, nrow - 1)] * a.lda + ch * 8) * 2);
    }
    const int fr = lane & 15, fq = lane >> 4, f = fr >> 1;
    c.ro0 = fr * 128 + ((fq ^ f) * 16);
    c.ro1 = fr * 128 + (((4 + fq) ^ f) * 16);
  }

  KGS_ACC_RESERVE();
  static_for<0, MA * NB>([](auto q) { accr::zero<decltype(q)::value>(); });
#pragma unroll
  for (int st = 0; st < NS; ++st) {
    const int kt = (st < c.nt ? st : c.nt - 1) * BK;
#pragma unroll
    for (int j = 0; j < ND; ++j) dma_any<BM, BN, X>(c, st, j, kt);
  }
  wait_vm<(NS - 1) * ND>();
  bar();
  Frag<MA, NB> f0, f1;
  {
    const char* pa = abase<BM, BN, 0>(c, 0);
    const char* pb = bbase<BM, BN, 0>(c, 0);
#pragma unroll
    for (int e = 0; e < S::NR; ++e) {
      const int x = rd_idx(KN::ORD, MA, NB, e);
      if (rd_isa(KN::ORD, MA, NB, e)) f0.a[x] = frag(pa + x * 2048); else f0.b[x] = frag(pb + x * 2048);
    }
  }
  __builtin_amdgcn_s_waitcnt(0xc07f);
  for (int t = 0; t < c.nt; t += NS) {
    kstep<BM, BN, 0, KN::B1, KN::R, KN::P, KN::ORD, X, NS>(c, f0, f1, t);
    if (NS == 2 || t + 1 < c.nt) kstep<BM, BN, 1, KN::B1, KN::R, KN::P, KN::ORD, X, NS>(c, f0, f1, t + 1);
    if constexpr (NS == 4) {
      if (t + 2 < c.nt) kstep<BM, BN, 2, KN::B1, KN::R, KN::P, KN::ORD, X, NS>(c, f0, f1, t + 2);
      if (t + 3 < c.nt) kstep<BM, BN, 3, KN::B1, KN::R, KN::P, KN::ORD, X, NS>(c, f0, f1, t + 3);
    }
  }
  asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
  asm volatile("s_nop 7\n\ts_nop 7\n\ts_nop 3" ::: "memory");  // MFMA -> v_accvgpr_read hazard

  const int fr = lane & 15, fq = lane >> 4;
  static_for<0, MA>([&](auto ic) {
    constexpr int i = decltype(ic)::value;
    const int lr = c.wr * (BM / 2) + i * 16 + fr;
    const long row = row0 + lr;
    const bool ok = lr < nrow;
    f32x4 v[NB];
    read_row<NB, i>(v);
    if constexpr (SPLIT) {
      float* part = (float*)a.C + ((long)slice * a.P + row) * a.N;
      if (ok)
#pragma unroll
        for (int n = 0; n < NB; ++n) *(f32x4*)(part + tn * BN + c.wc * (BN / 2) + n * 16 + fq * 4) = v[n];
    } else {
      unsigned short* crow = (unsigned short*)a.C + row * a.ldc;
      const float rw = GATED && ok ? a.roww[row] : 1.f;
      // GATED: out fragment p = gate fragment 4 (p / 2) + p % 2 with the up fragment two on
#pragma unroll
      for (int n = 0; n < (GATED ? NB / 2 : NB); n += 2) {
        uint2 o[2];
#pragma unroll
        for (int h = 0; h < 2; ++h) {
          float r[4];
          if constexpr (GATED) {
            const int ng = 4 * ((n + h) / 2) + (n + h) % 2;
#pragma unroll
            for (int e = 0; e < 4; ++e) r[e] = gated_weighted(v[ng][e], v[ng + 2][e], rw, a);
          } else {
#pragma unroll
            for (int e = 0; e < 4; ++e) r[e] = v[n + h][e];
          }
          o[h].x = pack_bf16x2(r[0], r[1]);
          o[h].y = pack_bf16x2(r[2], r[3]);
        }
        auto sx = __builtin_amdgcn_permlane16_swap(o[0].x, o[1].x, false, false);
        auto sy = __builtin_amdgcn_permlane16_swap(o[0].y, o[1].y, false, false);
        const int col0 = GATED ? tn * (BN / 2) + c.wc * (BN / 4) + n * 16 : tn * BN + c.wc * (BN / 2) + n * 16;
        if (ok) *(uint4*)(crow + col0 + (fq & 1) * 16 + (fq >> 1) * 8) = make_uint4(sx[0], sy[0], sx[1], sy[1]);
      }
    }
  });
}

// fp32: 64 x 64 tiles, 4 x 4 outputs per thread (gate and up side by side)
template <bool GATED>
__global__ __launch_bounds__(256) void grouped_f32(GroupedArgs a) {
  constexpr int TK = 16;
  const int ntn = (GATED ? a.N / 2 : a.N) / 64;
  if ((int)blockIdx.x >= *a.ntiles * ntn) return;
  const int4 tile = a.tiles[blockIdx.x / ntn];
  const int n0 = blockIdx.x % ntn * 64, tid = threadIdx.x, tx = tid & 15, ty = tid >> 4;
  __shared__ float as[TK][68], bs[2][TK][68];
  const float* B = (const float*)a.B + (long)tile.x * a.N * a.K;
  const int lr = tid >> 2, lk = (tid & 3) * 4;  // staging: row, first of 4 k
  const int ar = tile.y + min(lr, tile.z - 1);
  const float* ap = (const float*)a.A + (long)(GATED ? a.rows[ar] : ar) * a.lda + lk;
  const float* bp = B + (long)(n0 + lr) * a.K + lk;
  const float* up = bp + (long)(a.N / 2) * a.K;
  float g[4][4] = {}, u[4][4] = {};
  for (int k0 = 0; k0 < a.K; k0 += TK) {
    const f32x4 av = *(const f32x4*)(ap + k0), bv = *(const f32x4*)(bp + k0);
    f32x4 uv{};
    if constexpr (GATED) uv = *(const f32x4*)(up + k0);
    __syncthreads();
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      as[lk + i][lr] = av[i];
      bs[0][lk + i][lr] = bv[i];
      if constexpr (GATED) bs[1][lk + i][lr] = uv[i];
    }
    __syncthreads();
#pragma unroll
    for (int k = 0; k < TK; ++k) {
#pragma unroll
      for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          g[i][j] = __builtin_fmaf(as[k][4 * ty + i], bs[0][k][4 * tx + j], g[i][j]);
          if constexpr (GATED) u[i][j] = __builtin_fmaf(as[k][4 * ty + i], bs[1][k][4 * tx + j], u[i][j]);
        }
    }
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int r = 4 * ty + i;
    if (r >= tile.z) continue;
    float* cp = (float*)a.C + (long)(tile.y + r) * a.ldc + n0 + 4 * tx;
    const float rw = GATED ? a.roww[tile.y + r] : 1.f;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      if constexpr (GATED) {
        if (a.act == ACT_SILU) cp[j] = g[i][j] / (1.0f + expf(-g[i][j])) * u[i][j] * rw;
        else {
          const float gg = fminf(g[i][j] * rw, a.limit), uu = fminf(fmaxf(u[i][j] * rw, -a.limit), a.limit);
          cp[j] = gg / (1.0f + expf(-1.702f * gg)) * (uu + 1.0f);
        }
      } else cp[j] = g[i][j];
    }
  }
}

template <int ET>
int launch_route(const RouteArgs& a, size_t lds, hipStream_t s) {
  const size_t all = lds + 8 * RT * (a.ep + 1) * 4;
  if (all > 64 * 1024) return KGS_ERR_SHAPE;
  hipLaunchKernelGGL((route_mfma<ET>), dim3((a.T + RT - 1) / RT), dim3(512), all, s, a);
  return (int)hipGetLastError();
}

template <typename T>
int launch_plain(const RouteArgs& a, size_t lds, hipStream_t s) {
  if (lds > 160 * 1024) return KGS_ERR_SHAPE;
  if (lds > 64 * 1024) {
    const hipError_t e = hipFuncSetAttribute((const void*)route_plain<T>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    if (e != hipSuccess) return (int)e;
  }
  hipLaunchKernelGGL(route_plain<T>, dim3((a.T + RT - 1) / RT), dim3(256), lds, s, a);
  return (int)hipGetLastError();
}

int route(const RouteArgs& a, int f32, hipStream_t s) {
  const int zs = a.ep + 1;
  const size_t work = a.corr ? (size_t)RT * (a.groups + 2 * a.top) * 4 : 0;
  const size_t lds = ((size_t)RT * zs + a.E) * 4 + work, plain = lds + (a.corr ? (size_t)RT * zs * 4 : 0);
  if (f32) return launch_plain<float>(a, plain, s);
  if (a.ep <= 16) return launch_route<1>(a, lds, s);
  if (a.ep <= 32) return launch_route<2>(a, lds, s);
  if (a.ep == 64) return launch_route<4>(a, lds, s);
  return launch_plain<unsigned short>(a, plain, s);
}

}  // namespace moe
}  // namespace kgs

// Router logits of h [T, wp] with w [ep, wp] (wp % 256, ep % 16), the top choices per
// token (ids -1: a row whose slot is negative), their weights and their ranks;
// counts [E] must be zero and ends as the tokens of every expert.
KGS_EXPORT int kgs_moe_route(const void* h, long ldh, const void* w, const void* slots, void* counts, void* ids,
                             void* rank, void* weight, int T, int E, int ep, int wp, int top, int f32, hipStream_t s) {
  using namespace kgs::moe;
  if (T <= 0 || E <= 0 || E > 1024 || ep < E || ep % 16 || top <= 0 || top > E || wp <= 0 || wp % 256 || ldh < wp)
    return KGS_ERR_SHAPE;
  if (ldh % 8 || (((uintptr_t)h | (uintptr_t)w) & 15)) return KGS_ERR_ALIGN;
  RouteArgs a{h, ldh, w, (const int*)slots, (int*)counts, (int*)ids, (int*)rank, (float*)weight, T, E, ep, wp, top};
  return route(a, f32, s);
}

// The same with softmax scores over E experts and `extra` outputs that return their
// input: the `top` largest of score + corr [E + extra] among the best `keep` of `groups`
// groups of neighbours (by their largest), weights scale s / (sum s + 1e-20). ids -1 also
// for an extra output; ident [T]: the sum of a token's weights of those. gate [T]:
// sigmoid of router row E + extra. ident and gate may be null.
KGS_EXPORT int kgs_moe_route_softmax(const void* h, long ldh, const void* w, const void* slots, void* counts, void* ids,
                                     void* rank, void* weight, const void* corr, void* ident, void* gate, int T, int E,
                                     int extra, int groups, int keep, float scale, int ep, int wp, int top, int f32,
                                     hipStream_t s) {
  using namespace kgs::moe;
  const int EA = E + extra;
  if (T <= 0 || E <= 0 || extra < 0 || EA > 1024 || ep < EA + (gate ? 1 : 0) || ep % 16 || groups <= 0 || EA % groups ||
      keep <= 0 || keep > groups || top <= 0 || top > EA / groups * keep || wp <= 0 || wp % 256 || ldh < wp)
    return KGS_ERR_SHAPE;
  if (!corr) return KGS_ERR_ARG;
  if (ldh % 8 || (((uintptr_t)h | (uintptr_t)w) & 15)) return KGS_ERR_ALIGN;
  RouteArgs a{h, ldh, w, (const int*)slots, (int*)counts, (int*)ids, (int*)rank, (float*)weight, T, E, ep, wp, top,
              (const float*)corr, (float*)ident, (float*)gate, extra, groups, keep, scale};
  return route(a, f32, s);
}

KGS_EXPORT int kgs_moe_plan(const void* counts, const void* ids, const void* rank, const void* weight, void* pos,
                            void* rows, void* roww, void* tiles, void* ntiles, int T, int top, int E, int bm,
                            hipStream_t s) {
  using namespace kgs::moe;
  if (T <= 0 || top <= 0 || E <= 0 || E > 1024 || bm <= 0 || (long)T * top > 0x7fffffff) return KGS_ERR_SHAPE;
  PlanArgs a{(const int*)counts, (const int*)ids, (const int*)rank, (const float*)weight, (int*)pos, (int*)rows,
             (float*)roww, (int4*)tiles, (int*)ntiles, T * top, top, E, bm};
  hipLaunchKernelGGL(plan, dim3((T * top + 1023) / 1024), dim3(1024), 0, s, a);
  return (int)hipGetLastError();
}

// The experts' products over the sorted order. gated: C[p] = the gated product (act 0:
// clamped at limit, 1: silu) of A[rows[p]] with B [E][gate | up = N][K], N / 2 columns; else C[p] = B[e] A[p], nslice > 1: fp32
// partial products [slice][P][N] over K / nslice columns each. max_tiles: the most
// tiles of bm rows there can be.
KGS_EXPORT int kgs_moe_grouped(const void* A, long lda, const void* B, void* C, long ldc, const void* rows,
                               const void* roww, const void* tiles, const void* ntiles, int max_tiles, int bm, int T,
                               int P, int N, int K, int nslice, float limit, int act, int gated, int f32,
                               hipStream_t s) {
  using namespace kgs::moe;
  if (act != ACT_CLAMPED && act != ACT_SILU) return KGS_ERR_ARG;
  if (max_tiles <= 0 || T <= 0 || P <= 0 || N <= 0 || K <= 0 || nslice <= 0 || K % nslice) return KGS_ERR_SHAPE;
  const int kk = K / nslice, no = gated ? N / 2 : N;
  if (lda < K || (nslice == 1 && ldc < no) || (gated && nslice != 1)) return KGS_ERR_SHAPE;
  GroupedArgs a{A, B, C, (const int*)rows, (const float*)roww, (const int4*)tiles, (const int*)ntiles, lda,
                T, P, N, kk, (int)ldc, nslice, limit, act};
  if (f32) {
    if (bm != 64 || no % 64 || K % 16 || nslice != 1 || lda % 4) return KGS_ERR_SHAPE;
    const long g = (long)max_tiles * (no / 64);
    if (g > 0x7fffffff) return KGS_ERR_SHAPE;
    if (gated) hipLaunchKernelGGL(grouped_f32<true>, dim3((unsigned)g), dim3(256), 0, s, a);
    else hipLaunchKernelGGL(grouped_f32<false>, dim3((unsigned)g), dim3(256), 0, s, a);
    return (int)hipGetLastError();
  }
  if ((lda | ldc) % 8 || (((uintptr_t)A | (uintptr_t)B | (uintptr_t)C) & 15)) return KGS_ERR_ALIGN;
  // 32-bit byte offsets inside one buffer
  if ((long)T * lda * 2 > 0x7fffffff || 256l * lda * 2 > 0x7fffffff || 256l * K * 2 > 0x7fffffff) return KGS_ERR_SHAPE;
  const int bn = bm == 256 ? 256 : 128;
  if ((bm != 256 && bm != 128) || N % bn || kk % 128 || (gated && no % (bn / 2))) return KGS_ERR_SHAPE;
  const long g = (long)max_tiles * (N / bn) * nslice;
  if (g > 0x7fffffff) return KGS_ERR_SHAPE;
  const dim3 grid((unsigned)g), block(256);
  if (bm == 256) {
    if (nslice != 1) return KGS_ERR_ARG;
    if (gated) hipLaunchKernelGGL((grouped<256, 256, 2, true, false>), grid, block, 0, s, a);
    else hipLaunchKernelGGL((grouped<256, 256, 2, false, false>), grid, block, 0, s, a);
  } else if (gated) hipLaunchKernelGGL((grouped<128, 128, 4, true, false>), grid, block, 0, s, a);
  else if (nslice == 1) hipLaunchKernelGGL((grouped<128, 128, 4, false, false>), grid, block, 0, s, a);
  else hipLaunchKernelGGL((grouped<128, 128, 4, false, true>), grid, block, 0, s, a);
  return (int)hipGetLastError();
}
