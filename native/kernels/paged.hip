// Softmax attention over head pages (talking.hip's page layout: K and V of one key head
// in MFMA fragment order) for gfx950: grouped key heads, any key and value sizes, causal,
// optionally chunked: with chunk size c a query at position i sees the keys j <= i of its
// own chunk, floor(j / c) = floor(i / c), so it reads only the pages from its chunk's
// first key on.
//
//   rows   decoded tokens and short portions: one query token's heads of a key head are
//          the columns of S^T = K Q^T. K lane 16 q + n of a page's half kt holds token
//          2 n + kt, so a lane's 8 scores are tokens 8 q .. of one head, which is the
//          operand layout of O^T = V^T P^T: nothing moves between lanes but the maximum.
//   tiles  prompt portions: 128 (query, head of the group) rows per workgroup, 32 per
//          wave, S^T on 32x32x16 MFMAs. Row i of a K tile is token i with bits 2 and 3
//          swapped, so that the scores of a k-step come out as the 8 consecutive tokens
//          V's fragments hold.
//   plain  fp32, and sizes the others do not take.
//
// Differential heads (two maps): a head has two queries and a key head two keys, each half of
// the dkp columns; both maps' softmaxes weigh the same values, and the head's output is
//   o = a1 - lam a2,   o <- post o / sqrt(mean o^2 + eps)  over its vdim values.
//   rows   the maps are columns: 8 heads' first and 8 heads' second queries, each zero in the
//          other map's dims, so both maps' scores add up in one accumulator and V is
//          multiplied once.
//   tiles  the maps are waves: 64 (query, head) rows, two waves per map; the second map's
//          waves hand their results to the first one's through LDS.
//
// Pages go to LDS (tiles) by DMA as they are: fragment order is free of bank conflicts.
#include "kgs_common.h"

namespace kgs {
namespace paged {

typedef float f32x16 __attribute__((ext_vector_type(16)));
typedef unsigned u32x4 __attribute__((ext_vector_type(4)));

constexpr int PAGE = 32;
constexpr float NEG = -1.0e30f;
constexpr float RESCALE = 8.0f;  // log2 units a score may exceed the running maximum by
constexpr int ROWS = 128;        // of a tile

__device__ __forceinline__ int k_at(int tok, int d, int nk) {
  return (((tok & 1) * nk + (d >> 5)) * 64 + ((d >> 3) & 3) * 16 + (tok >> 1)) * 8 + (d & 7);
}
__device__ __forceinline__ int v_at(int tok, int d) {
  return ((d >> 4) * 64 + (tok >> 3) * 16 + (d & 15)) * 8 + (tok & 7);
}

struct Args {
  const void* q;       // [T, ldq], head h at column h dkp
  long ldq;
  const void* pages;
  void* o;             // [T, ldo], head h at column h dvp
  long ldo;
  const int* bt;       // [sequences, W]
  int W;
  const int* tok_seq;  // rows: per query its block-table row and its position
  const int* tok_pos;
  const int* rows;     // its batch row, or null: the same
  const int4* items;   // tiles: (first batch row, block-table row, position, queries)
  float* po;           // partial results of split rows: [row, split][heads][dvp]
  float* pml;          // [row, split][heads][2]
  float sl2;           // scale log2(e)
  int chunk;           // 0: none
  int H, G, R, dkp, dvp, nsplit;
  int maps, vdim;      // 1, or 2: differential heads
  float lam, post, eps;
};

__device__ __forceinline__ int first_key(const Args& a, int pos) { return a.chunk ? pos - pos % a.chunk : 0; }

// ------------------------------------------------------------------------ rows
// grid: row x key head x 16 (8) heads of its group x split; four waves take the split's pages in turn
template <int NK, int ND, int MAPS = 1>
__global__ __launch_bounds__(256, 2) void attn_rows(Args a) {
  const int lane = threadIdx.x & 63, w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), n = lane & 15, q = lane >> 4;
  constexpr int HT = 16 / MAPS;  // heads of a workgroup, MAPS columns each
  constexpr bool AHEAD = 2 * NK + ND <= 16;  // the next page's fragments fit in registers
  const int nht = (a.R + HT - 1) / HT;
  int id = blockIdx.x;
  const int sp = id % a.nsplit;
  id /= a.nsplit;
  const int ht = id % nht;
  id /= nht;
  const int g = id % a.G, row = id / a.G;
  const int h0 = g * a.R + HT * ht, nh = min(HT, a.R - HT * ht);
  const int pos = a.tok_pos[row], lo = first_key(a, pos), fp = lo / PAGE, npage = pos / PAGE + 1 - fp;
  const int per = (npage + a.nsplit - 1) / a.nsplit, p0 = fp + sp * per, p1 = min(fp + npage, p0 + per);
  const int* bt = a.bt + (long)a.tok_seq[row] * a.W;
  const long brow = a.rows ? a.rows[row] : row;
  __shared__ __attribute__((aligned(16))) float lo_acc[4][ND * 256];  // [wave][dim][head]
  __shared__ float lml[4][16][2];

  bf16x8 qf[NK];
  {
    const unsigned short* qp = (const unsigned short*)a.q + brow * a.ldq + (long)(h0 + min(n % HT, nh - 1)) * (NK * 32) + 8 * q;
#pragma unroll
    for (int ks = 0; ks < NK; ++ks) {
      qf[ks] = *(const bf16x8*)(qp + 32 * ks);
      if (MAPS == 2 && n / HT != ks / (NK / MAPS)) qf[ks] = bf16x8{};
    }
  }
  f32x4 acc[ND];
#pragma unroll
  for (int d = 0; d < ND; ++d) acc[d] = f32x4{};
  float m = NEG, l = 0.f;

  const long hpage = PAGE * (NK * 32 + ND * 16);
  struct Frags {
    bf16x8 k[2 * NK], v[ND];
  };
  auto load = [&](int p, Frags& f) {
    const unsigned short* s = (const unsigned short*)a.pages + ((long)bt[p] * a.G + g) * hpage + 8 * lane;
#pragma unroll
    for (int i = 0; i < 2 * NK; ++i) f.k[i] = __builtin_nontemporal_load((const bf16x8*)(s + 512 * i));
#pragma unroll
    for (int i = 0; i < ND; ++i) f.v[i] = __builtin_nontemporal_load((const bf16x8*)(s + 1024 * NK + 512 * i));
  };
  auto work = [&](int p, const Frags& f) {
    f32x4 S[2];
#pragma unroll
    for (int kt = 0; kt < 2; ++kt) {
      S[kt] = f32x4{};
#pragma unroll
      for (int ks = 0; ks < NK; ++ks) S[kt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(f.k[kt * NK + ks], qf[ks], S[kt], 0, 0, 0);
    }
    const int tok0 = p * PAGE + 8 * q;
    const bool edge = p * PAGE < lo || p * PAGE + PAGE - 1 > pos;
    float mx = m;
#pragma unroll
    for (int kt = 0; kt < 2; ++kt)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int tok = tok0 + 2 * r + kt;
        S[kt][r] *= a.sl2;
        if (edge && (tok < lo || tok > pos)) S[kt][r] = NEG;
        mx = fmaxf(mx, S[kt][r]);
      }
    if (__any(mx > m + RESCALE)) {
      mx = xor32_max(xor16_max(mx));
      const float al = __builtin_amdgcn_exp2f(m - mx);
      m = mx;
      l *= al;
#pragma unroll
      for (int d = 0; d < ND; ++d) acc[d] *= al;
    }
    u32x4 pk;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const float x = __builtin_amdgcn_exp2f(S[0][r] - m), y = __builtin_amdgcn_exp2f(S[1][r] - m);
      l += x + y;
      pk[r] = pack_bf16x2(x, y);
    }
    const bf16x8 pf = __builtin_bit_cast(bf16x8, pk);
#pragma unroll
    for (int d = 0; d < ND; ++d) acc[d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(f.v[d], pf, acc[d], 0, 0, 0);
  };
  int p = p0 + w;
  if (p < p1) {
    Frags f0;
    if constexpr (AHEAD) {
      Frags f1;
      load(p, f0);
      for (; p < p1; p += 8) {
        const bool more = p + 4 < p1;
        if (more) load(p + 4, f1);
        work(p, f0);
        if (!more) break;
        if (p + 8 < p1) load(p + 8, f0);
        work(p + 4, f1);
      }
    } else {
      for (; p < p1; p += 4) {
        load(p, f0);
        work(p, f0);
      }
    }
  }

  l = xor32_sum(xor16_sum(l));
#pragma unroll
  for (int d = 0; d < ND; ++d)
#pragma unroll
    for (int r = 0; r < 4; ++r) lo_acc[w][(16 * d + 4 * q + r) * 16 + n] = acc[d][r];
  if (q == 0) lml[w][n][0] = m, lml[w][n][1] = l;
  __syncthreads();
  constexpr int DV = ND * 16;
  // column c, dim d: the waves' sum y and its weight L
  auto gather = [&](int c, int d, float& y, float& L, float& M) {
    M = lml[0][c][0];
#pragma unroll
    for (int x = 1; x < 4; ++x) M = fmaxf(M, lml[x][c][0]);
    y = 0.f, L = 0.f;
#pragma unroll
    for (int x = 0; x < 4; ++x) {
      const float f = __builtin_amdgcn_exp2f(lml[x][c][0] - M);
      L = __builtin_fmaf(f, lml[x][c][1], L);
      y = __builtin_fmaf(f, lo_acc[x][d * 16 + c], y);
    }
  };
  if (a.nsplit > 1) {
    for (int i = threadIdx.x; i < nh * MAPS * DV; i += 256) {
      const int j = i / DV, d = i - j * DV;  // head j / MAPS, map j % MAPS
      float y, L, M;
      gather(j / MAPS + HT * (j % MAPS), d, y, L, M);
      const long at = (((long)row * a.nsplit + sp) * a.H + h0) * MAPS + j;
      a.po[at * DV + d] = y;
      if (d == 0) a.pml[2 * at] = M, a.pml[2 * at + 1] = L;
    }
  } else if constexpr (MAPS == 1) {
    for (int i = threadIdx.x; i < nh * DV; i += 256) {
      const int c = i / DV, d = i - c * DV;
      float y, L, M;
      gather(c, d, y, L, M);
      ((unsigned short*)a.o)[brow * a.ldo + (long)(h0 + c) * DV + d] = f2bf(y / L);
    }
  } else {
    __shared__ float diff[HT][DV];
    for (int i = threadIdx.x; i < nh * DV; i += 256) {
      const int c = i / DV, d = i - c * DV;
      float y1, L1, y2, L2, M;
      gather(c, d, y1, L1, M);
      gather(c + HT, d, y2, L2, M);
      diff[c][d] = y1 / L1 - a.lam * (y2 / L2);
    }
    __syncthreads();
    for (int c = w; c < nh; c += 4) {
      float ss = 0.f;
#pragma unroll
      for (int d = lane; d < DV; d += 64) ss = __builtin_fmaf(diff[c][d], diff[c][d], ss);
      const float f = a.post / sqrtf(wave_sum(ss) / a.vdim + a.eps);
#pragma unroll
      for (int d = lane; d < DV; d += 64)
        ((unsigned short*)a.o)[brow * a.ldo + (long)(h0 + c) * DV + d] = f2bf(diff[c][d] * f);
    }
  }
}

// splits of one (row, head) -> its output; an empty split has maximum NEG and sum 0
constexpr int MERGE_DIMS = 2;  // 64 value dims each (MFMA sizes)
template <int MAPS>
__global__ __launch_bounds__(64) void merge(Args a) {
  const int row = blockIdx.x / a.H, h = blockIdx.x - row * a.H;
  const long brow = a.rows ? a.rows[row] : row;
  const int lane = threadIdx.x, step = a.H * MAPS;  // columns of a split
  float o[MERGE_DIMS] = {};
#pragma unroll
  for (int map = 0; map < MAPS; ++map) {
    const long at = (long)row * a.nsplit * step + h * MAPS + map;
    // one lane per split (at most 64): its factor, and the sum of all
    const float* ml = a.pml + 2 * (at + (long)min(lane, a.nsplit - 1) * step);
    const float m = lane < a.nsplit ? ml[0] : NEG, l = lane < a.nsplit ? ml[1] : 0.f;
    float M = m;
#pragma unroll
    for (int x = 1; x < 64; x <<= 1) M = fmaxf(M, __shfl_xor(M, x));
    const float f = __builtin_amdgcn_exp2f(m - M), inv = (map ? -a.lam : 1.0f) / wave_sum(f * l);
#pragma unroll
    for (int k = 0; k < MERGE_DIMS; ++k) {
      const int d = 64 * k + lane;
      const float* p = a.po + at * a.dvp + min(d, a.dvp - 1);
      float y = 0.f;
      for (int s = 0; s < a.nsplit; s += 8)  // eight loads in flight; past the last split the factor is 0
#pragma unroll
        for (int i = 0; i < 8; ++i)
          y = __builtin_fmaf(__shfl(f, s + i), p[(long)min(s + i, a.nsplit - 1) * step * a.dvp], y);
      o[k] = d < a.dvp ? __builtin_fmaf(y, inv, o[k]) : 0.f;
    }
  }
  float f = 1.0f;
  if constexpr (MAPS == 2) {
    float ss = 0.f;
#pragma unroll
    for (int k = 0; k < MERGE_DIMS; ++k) ss = __builtin_fmaf(o[k], o[k], ss);
    f = a.post / sqrtf(wave_sum(ss) / a.vdim + a.eps);
  }
#pragma unroll
  for (int k = 0; k < MERGE_DIMS; ++k) {
    const int d = 64 * k + lane;
    if (d < a.dvp) ((unsigned short*)a.o)[brow * a.ldo + (long)h * a.dvp + d] = f2bf(o[k] * f);
  }
}

// ----------------------------------------------------------------------- tiles
// grid: item x key head. Row i of an item is query i / R, head i % R of the group. DK: dims of
// one map.
template <int DK, int DV, int MAPS = 1>
__global__ __launch_bounds__(256, 2) __attribute__((amdgpu_waves_per_eu(2, 2))) void attn_tiles(Args a) {
  constexpr int NK = DK / 16, ND = DV / 32, PB = PAGE * (MAPS * DK + DV) * 2;  // k-steps, dim tiles, bytes of a head's page
  constexpr int PG = 4 * PB <= 80 * 1024 ? 2 : 1;  // pages of a tile: two workgroups per CU
  constexpr int NCH = PG * PB / 1024;              // its 1 KB pieces
  __shared__ __attribute__((aligned(1024))) char smem[2][PG * PB];
  const int lane = threadIdx.x & 63, w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), l32 = lane & 31, hh = lane >> 5;
  const int item = blockIdx.x / a.G, g = blockIdx.x - item * a.G;
  const int4 it = a.items[item];
  const int nrow = it.w * a.R;
  const int* bt = a.bt + (long)it.y * a.W;
  const int map = MAPS == 2 ? w >> 1 : 0, wr = 32 * (MAPS == 2 ? w & 1 : w);  // this wave's map and first row
  const int ri = min(wr + l32, nrow - 1), ti = ri / a.R, h = g * a.R + ri - ti * a.R;
  const int qpos = it.z + ti, qlo = first_key(a, qpos);
  // this wave's first and last query
  const int w0 = it.z + min(wr, nrow - 1) / a.R, w1 = it.z + min(wr + 31, nrow - 1) / a.R;
  const int wlo0 = first_key(a, w0), wlo1 = first_key(a, w1);
  const bool active = wr < nrow;

  bf16x8 qf[NK];
  {
    const bf16x8* qp = (const bf16x8*)((const unsigned short*)a.q + (long)(it.x + ti) * a.ldq + ((long)h * MAPS + map) * DK + 8 * hh);
#pragma unroll
    for (int ks = 0; ks < NK; ++ks) qf[ks] = qp[2 * ks];
  }
  const int fp = first_key(a, it.z) / PAGE, lp = (it.z + it.w - 1) / PAGE, ntile = (lp - fp) / PG + 1;
  const unsigned short* base = (const unsigned short*)a.pages + (long)g * (PB / 2) + 8 * lane;
  auto dma = [&](int j, int buf) {
    const int pa = bt[fp + PG * j], pb = PG == 2 ? bt[min(fp + 2 * j + 1, lp)] : 0;  // past the last page: it again, masked
#pragma unroll
    for (int i = 0; i < NCH / 4; ++i) {
      const int ch = NCH / 4 * w + i, half = PG == 2 && ch >= NCH / 2;
      const unsigned short* s = base + (long)(half ? pb : pa) * a.G * (PB / 2) + (ch - half * (NCH / 2)) * 512;
      glds16(s, smem[buf] + 1024 * ch);
    }
  };
  dma(0, 0);
  __builtin_amdgcn_s_waitcnt(0x0f70);  // vmcnt(0)
  __syncthreads();

  f32x16 o[ND];
#pragma unroll
  for (int d = 0; d < ND; ++d) o[d] = f32x16{};
  float m = NEG, l = 0.f;
  const float sl2 = a.sl2;
  const int tk = (l32 & ~12) | ((l32 & 4) << 1) | ((l32 & 8) >> 1);  // bits 2 and 3 swapped
  const int koff = (((tk & 1) * MAPS + map) * (DK / 32) * 64 + hh * 16 + (tk >> 1)) * 16;
  const int voff = ((l32 >> 4) * 64 + hh * 16 + (l32 & 15)) * 16;

  for (int j = 0; j < ntile; ++j) {
    const int buf = j & 1;
    if (j + 1 < ntile) dma(j + 1, buf ^ 1);  // released by the previous tile's barrier
    const int kv0 = (fp + PG * j) * PAGE;
    if (active && kv0 <= w1 && kv0 + PG * PAGE > wlo0) {
      const char* sm = smem[buf];
      bf16x8 kf[PG][NK];
#pragma unroll
      for (int t = 0; t < PG; ++t)
#pragma unroll
        for (int ks = 0; ks < NK; ++ks)  // dims 16 ks + 8 hh ..
          kf[t][ks] = *(const bf16x8*)(sm + t * PB + koff + ((ks >> 1) * 64 + (ks & 1) * 32) * 16);
      __builtin_amdgcn_sched_barrier(0);
      f32x16 s[PG];
#pragma unroll
      for (int t = 0; t < PG; ++t) {
        s[t] = f32x16{};
#pragma unroll
        for (int ks = 0; ks < NK; ++ks) s[t] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(kf[t][ks], qf[ks], s[t], 0, 0, 0);
      }
      bf16x8 vf[ND][PG][2];
      auto read_v = [&](int d) {
#pragma unroll
        for (int t = 0; t < PG; ++t)
#pragma unroll
          for (int sp = 0; sp < 2; ++sp)
            vf[d][t][sp] = *(const bf16x8*)(sm + t * PB + PAGE * MAPS * DK * 2 + voff + (2 * d * 64 + 2 * sp * 16) * 16);
      };
      read_v(0);
      read_v(1);
      __builtin_amdgcn_sched_barrier(0);
      if (kv0 + PG * PAGE - 1 > w0 || kv0 < wlo1) {
#pragma unroll
        for (int t = 0; t < PG; ++t)
#pragma unroll
          for (int r = 0; r < 16; ++r) {
            const int kv = kv0 + 32 * t + 16 * (r >> 3) + 8 * hh + (r & 7);
            if (kv > qpos || kv < qlo) s[t][r] = NEG;
          }
      }
      float mx = m;
#pragma unroll
      for (int t = 0; t < PG; ++t)
#pragma unroll
        for (int r = 0; r < 16; ++r) mx = fmaxf(mx, s[t][r]);
      mx = xor32_max(mx);
      const bool grow = (mx - m) * sl2 > RESCALE;
      if (__any(grow)) {
        const float mn = grow ? mx : m;
        const float alpha = __builtin_amdgcn_exp2f((m - mn) * sl2);
        m = mn;
        l *= alpha;
#pragma unroll
        for (int d = 0; d < ND; ++d) o[d] *= alpha;
      }
      const float msl = m == NEG ? 0.f : m * sl2;  // a row that has seen no key yet: weights 0
#pragma unroll
      for (int t = 0; t < PG; ++t)
#pragma unroll
        for (int r = 0; r < 16; ++r) {
          const float p = __builtin_amdgcn_exp2f(__builtin_fmaf(s[t][r], sl2, -msl));
          s[t][r] = p;
          l += p;
        }
      bf16x8 pf[PG][2];
#pragma unroll
      for (int t = 0; t < PG; ++t) {
        pf[t][0] = pack_bf16x8(s[t], 0);
        pf[t][1] = pack_bf16x8(s[t], 8);
      }
      if constexpr (ND == 4) {
        read_v(2);
        read_v(3);
      }
#pragma unroll
      for (int d = 0; d < ND; ++d)
#pragma unroll
        for (int t = 0; t < PG; ++t)
#pragma unroll
          for (int sp = 0; sp < 2; ++sp)
            o[d] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf[d][t][sp], pf[t][sp], o[d], 0, 0, 0);
    }
    __builtin_amdgcn_s_waitcnt(0x0f70);  // vmcnt(0): the next tile has landed
    __syncthreads();
  }
  l = xor32_sum(l);
  float inv = 1.0f / l;
  if constexpr (MAPS == 2) {
    static_assert(2 * ND * 16 * 64 * 4 <= (int)sizeof(smem), "the second map's results fit in the page buffers");
    float* xch = (float*)smem + (w & 1) * (ND * 16 * 64) + lane;
    if (map)
#pragma unroll
      for (int d = 0; d < ND; ++d)
#pragma unroll
        for (int r = 0; r < 16; ++r) xch[(16 * d + r) * 64] = o[d][r] * inv;
    __syncthreads();
    if (map) return;
    float ss = 0.f;
#pragma unroll
    for (int d = 0; d < ND; ++d)
#pragma unroll
      for (int r = 0; r < 16; ++r) {
        o[d][r] = __builtin_fmaf(-a.lam, xch[(16 * d + r) * 64], o[d][r] * inv);
        ss = __builtin_fmaf(o[d][r], o[d][r], ss);
      }
    inv = a.post / sqrtf(xor32_sum(ss) / a.vdim + a.eps);
  }
  if (wr + l32 >= nrow) return;
  unsigned short* op = (unsigned short*)a.o + (long)(it.x + ti) * a.ldo + (long)h * DV;
#pragma unroll
  for (int d = 0; d < ND; ++d)
#pragma unroll
    for (int r4 = 0; r4 < 4; ++r4) {
      uint2 pk;
      pk.x = pack_bf16x2(o[d][4 * r4 + 0] * inv, o[d][4 * r4 + 1] * inv);
      pk.y = pack_bf16x2(o[d][4 * r4 + 2] * inv, o[d][4 * r4 + 3] * inv);
      *(uint2*)(op + 32 * d + 8 * r4 + 4 * hh) = pk;
    }
}

// ----------------------------------------------------------------------- plain
template <typename T>
__device__ __forceinline__ float ld(const T* p) {
  if constexpr (sizeof(T) == 2) return bf2f(*(const unsigned short*)p);
  else return *p;
}

constexpr int PLAIN_DIMS = 4;  // value dims per thread

// one workgroup per (row, head), 256 keys at a time
template <typename T>
__global__ __launch_bounds__(256) void attn_plain(Args a) {
  extern __shared__ float lds[];  // [dkp] query, [256] weights, [4] reduction
  const int tid = threadIdx.x, row = blockIdx.x / a.H, h = blockIdx.x - row * a.H, g = h / a.R;
  const int pos = a.tok_pos[row], lo = first_key(a, pos);
  const int* bt = a.bt + (long)a.tok_seq[row] * a.W;
  const long brow = a.rows ? a.rows[row] : row, per = (long)PAGE * (a.dkp + a.dvp);
  const int seg = a.dkp / a.maps;
  float* qs = lds;
  float* P = lds + seg;
  float* red = P + 256;
  float res[PLAIN_DIMS] = {};
  for (int map = 0; map < a.maps; ++map) {
    __syncthreads();  // the other map's query is used
    for (int d = tid; d < seg; d += 256) qs[d] = ld((const T*)a.q + brow * a.ldq + (long)h * a.dkp + map * seg + d) * a.sl2;
    float m = NEG, l = 0.f, o[PLAIN_DIMS] = {};
    for (int k0 = lo; k0 <= pos; k0 += 256) {
      __syncthreads();  // the query is there; the last weights are used
      const int k = k0 + tid;
      float s = NEG;
      if (k <= pos) {
        const T* kp = (const T*)a.pages + ((long)bt[k / PAGE] * a.G + g) * per;
        s = 0.f;
        for (int d = 0; d < seg; ++d) s = __builtin_fmaf(qs[d], ld(kp + k_at(k % PAGE, map * seg + d, a.dkp / 32)), s);
      }
      float mx = s;
#pragma unroll
      for (int x = 1; x < 64; x <<= 1) mx = fmaxf(mx, __shfl_xor(mx, x));
      if ((tid & 63) == 0) red[tid >> 6] = mx;
      __syncthreads();
      mx = fmaxf(fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3])), m);
      const float al = exp2f(m - mx), p = k <= pos ? exp2f(s - mx) : 0.f;
      m = mx;
      P[tid] = p;
      l *= al;
      __syncthreads();
      const int nk = min(256, pos + 1 - k0);
      for (int i = 0; i < nk; ++i) l += P[i];
#pragma unroll
      for (int j = 0; j < PLAIN_DIMS; ++j) {
        const int d = tid + 256 * j;
        if (d >= a.dvp) break;
        float y = o[j] * al;
        for (int i = 0; i < nk; ++i) {
          const T* vp = (const T*)a.pages + ((long)bt[(k0 + i) / PAGE] * a.G + g) * per + PAGE * a.dkp;
          y = __builtin_fmaf(P[i], ld(vp + v_at((k0 + i) % PAGE, d)), y);
        }
        o[j] = y;
      }
    }
#pragma unroll
    for (int j = 0; j < PLAIN_DIMS; ++j) res[j] = __builtin_fmaf(map ? -a.lam : 1.0f, o[j] / l, res[j]);
  }
  float f = 1.0f;
  if (a.maps == 2) {
    float ss = 0.f;
#pragma unroll
    for (int j = 0; j < PLAIN_DIMS; ++j) ss = __builtin_fmaf(res[j], res[j], ss);
    ss = wave_sum(ss);
    __syncthreads();
    if ((tid & 63) == 0) red[tid >> 6] = ss;
    __syncthreads();
    f = a.post / sqrtf((red[0] + red[1] + red[2] + red[3]) / a.vdim + a.eps);
  }
#pragma unroll
  for (int j = 0; j < PLAIN_DIMS; ++j) {
    const int d = tid + 256 * j;
    if (d >= a.dvp) break;
    const float y = res[j] * f;
    T* p = (T*)a.o + brow * a.ldo + (long)h * a.dvp + d;
    if constexpr (sizeof(T) == 2) *p = f2bf(y);
    else *p = y;
  }
}

template <int NK, int ND, int MAPS>
void run_rows(const Args& a, int nrows, hipStream_t s) {
  constexpr int HT = 16 / MAPS;
  hipLaunchKernelGGL((attn_rows<NK, ND, MAPS>), dim3((unsigned)(nrows * a.G * ((a.R + HT - 1) / HT) * a.nsplit)), dim3(256),
                     0, s, a);
  if (a.nsplit > 1) hipLaunchKernelGGL(merge<MAPS>, dim3((unsigned)(nrows * a.H)), dim3(64), 0, s, a);
}
template <int MAPS>
void run_rows(const Args& a, int nrows, hipStream_t s) {
  if (a.dkp == 64 * MAPS) a.dvp == 64 ? run_rows<2 * MAPS, 4, MAPS>(a, nrows, s) : run_rows<2 * MAPS, 8, MAPS>(a, nrows, s);
  else a.dvp == 64 ? run_rows<4 * MAPS, 4, MAPS>(a, nrows, s) : run_rows<4 * MAPS, 8, MAPS>(a, nrows, s);
}
template <int MAPS>
void run_tiles(const Args& a, int nitems, hipStream_t s) {
  const dim3 grid((unsigned)(nitems * a.G));
  auto fn = a.dkp == 64 * MAPS ? (a.dvp == 64 ? attn_tiles<64, 64, MAPS> : attn_tiles<64, 128, MAPS>)
                               : (a.dvp == 64 ? attn_tiles<128, 64, MAPS> : attn_tiles<128, 128, MAPS>);
  hipLaunchKernelGGL(fn, grid, dim3(256), 0, s, a);
}

int check(const Args& a, int n) {
  if (n <= 0 || a.H <= 0 || a.G <= 0 || a.H % a.G || a.dkp <= 0 || a.dvp <= 0 || a.dkp % 32 || a.dvp % 16 || a.W <= 0 ||
      a.chunk < 0 || a.ldq < (long)a.H * a.dkp || a.ldo < (long)a.H * a.dvp || (long)n * a.H > 0x7fffffff)
    return KGS_ERR_SHAPE;
  if (!(a.sl2 > 0.f) || (a.maps != 1 && a.maps != 2)) return KGS_ERR_ARG;
  if (a.dkp % (32 * a.maps) || (a.maps == 2 && (a.vdim <= 0 || a.vdim > a.dvp))) return KGS_ERR_SHAPE;
  if (a.ldq % 8 || a.ldo % 8 || (((uintptr_t)a.q | (uintptr_t)a.o | (uintptr_t)a.pages) & 15)) return KGS_ERR_ALIGN;
  return KGS_OK;
}

bool mfma(const Args& a) {
  return (a.dkp == 64 * a.maps || a.dkp == 128 * a.maps) && (a.dvp == 64 || a.dvp == 128);
}

}  // namespace paged
}  // namespace kgs

// nrows query tokens (batch row rows[i], or i), each over its sequence's pages up to its
// position, from its chunk's first key on (chunk 0: from 0). maps 2: differential heads, dkp
// holds both maps; lam, post, vdim, eps as at the top. bf16 with 64 or 128 dims per map and dvp
// 64 or 128, split over the pages nsplit <= 64 times (po, pml: partial results, maps columns per
// head); plain != 0 (or fp32): any sizes, dvp up to 1024.
KGS_EXPORT int kgs_paged_rows(const void* q, long ldq, const void* pages, void* o, long ldo, const void* bt, int W,
                              const void* tok_seq, const void* tok_pos, const void* rows, void* po, void* pml, float scale,
                              int chunk, int nrows, int H, int G, int dkp, int dvp, int maps, int vdim, float lam,
                              float post, float eps, int nsplit, int plain, int f32, hipStream_t s) {
  using namespace kgs::paged;
  Args a{q, ldq, pages, o, ldo, (const int*)bt, W, (const int*)tok_seq, (const int*)tok_pos, (const int*)rows, nullptr,
         (float*)po, (float*)pml, scale * 1.4426950408889634f, chunk, H, G, G ? H / G : 0, dkp, dvp, nsplit,
         maps, vdim, lam, post, eps};
  if (int rc = check(a, nrows)) return rc;
  if (plain || f32) {
    if (dvp > 256 * PLAIN_DIMS || dkp > 8192) return KGS_ERR_SHAPE;
    const size_t lds = (dkp / maps + 260) * 4;
    if (f32) hipLaunchKernelGGL(attn_plain<float>, dim3(nrows * H), dim3(256), lds, s, a);
    else hipLaunchKernelGGL(attn_plain<unsigned short>, dim3(nrows * H), dim3(256), lds, s, a);
    return (int)hipGetLastError();
  }
  if (!mfma(a)) return KGS_ERR_ARG;
  if (nsplit <= 0 || nsplit > 64 || (nsplit > 1 && (!po || !pml)) || (long)nrows * H * nsplit > 0x7fffffff) return KGS_ERR_SHAPE;
  maps == 2 ? run_rows<2>(a, nrows, s) : run_rows<1>(a, nrows, s);
  return (int)hipGetLastError();
}

// Prompt portions: nitems blocks of consecutive queries (first batch row, block-table row,
// position of the first, queries), queries x heads per key head <= 128 / maps in each, as
// kgs_paged_rows. bf16, 64 or 128 dims per map, dvp 64 or 128.
KGS_EXPORT int kgs_paged_tiles(const void* q, long ldq, const void* pages, void* o, long ldo, const void* bt, int W,
                               const void* items, int nitems, float scale, int chunk, int H, int G, int dkp, int dvp,
                               int maps, int vdim, float lam, float post, float eps, hipStream_t s) {
  using namespace kgs::paged;
  Args a{};
  a.q = q, a.ldq = ldq, a.pages = pages, a.o = o, a.ldo = ldo, a.bt = (const int*)bt, a.W = W;
  a.items = (const int4*)items, a.sl2 = scale * 1.4426950408889634f, a.chunk = chunk;
  a.H = H, a.G = G, a.R = G ? H / G : 0, a.dkp = dkp, a.dvp = dvp, a.nsplit = 1;
  a.maps = maps, a.vdim = vdim, a.lam = lam, a.post = post, a.eps = eps;
  if (int rc = check(a, nitems)) return rc;
  if (!mfma(a) || a.R > ROWS / maps) return KGS_ERR_ARG;
  if ((uintptr_t)items & 15) return KGS_ERR_ALIGN;
  maps == 2 ? run_tiles<2>(a, nitems, s) : run_tiles<1>(a, nitems, s);
  return (int)hipGetLastError();
}
