// Talking-heads attention for gfx950: before the softmax every head's score becomes
// a learned mixture of all heads' scores,
//
//   s_h(i, j) = sum_g talk[h, g] (temp_g scale q_g(i) . k_g(j) + rel_g[i - j])
//
// over a paged cache with grouped key / value heads, any key and value sizes, causal,
// with `1 +` in the softmax's denominator. Scores live in log2 units: sc[g] =
// temp scale log2(e), and the mixed distance bias is a table per distance, bias[n][h]
// = log2(e) sum_g talk[h, g] rel_g[n], whose last row serves every distance from
// its number on.
//
// The mixture is an MFMA over heads. talk is exact in bf16; a score enters as
// three bf16 parts (truncated, truncated, rest) that together hold its 24 bits, so
// the product is an fp32 one. What makes it cheap is that no score leaves the
// registers for it:
//   rows   (decoded tokens, short portions) S = q K^T with heads on the MFMA's rows
//          leaves a lane 4 heads of one key; an MFMA contracts in any order both
//          operands share, so those registers are its operand as they are, and with
//          talk on the other side the mixed scores come out as keys x heads, which is
//          the operand layout of P V.
//   tiles  (prompt portions) rows are 4 queries x 4 heads of one key head, so lane
//          group q holds query q; a 4 x 4 transpose between lane groups and registers
//          (two half-swaps) turns that into lane group q = heads 4q.. of one query.
//
// Page of one key head: K [kt 2][ks][lane][8] then V [dt][lane][8] bf16, in MFMA
// fragment order: K lane 16 q + n of (kt, ks): token 2n + kt, dims 32 ks + 8q ..;
// V lane 16 q + n of dt: dim 16 dt + n, tokens 8q .. (fp32: the same order).
//
// The running maximum starts at 0, the score of the `1 +`, so it never needs a
// first tile; each row's sum gets 2^(0 - max) once, at the end.
#include "kgs_common.h"

namespace kgs {
namespace talking {

constexpr int PAGE = 32;
constexpr float NEG = -1.0e30f;
constexpr float RESCALE = 8.0f;  // log2 units a score may exceed the running maximum by

__device__ __forceinline__ int k_at(int tok, int d, int nk) {
  return (((tok & 1) * nk + (d >> 5)) * 64 + ((d >> 3) & 3) * 16 + (tok >> 1)) * 8 + (d & 7);
}
__device__ __forceinline__ int v_at(int tok, int d) {
  return ((d >> 4) * 64 + (tok >> 3) * 16 + (d & 15)) * 8 + (tok & 7);
}

// three bf16 parts of an fp32 value, each in the upper half of its word; exact
__device__ __forceinline__ void split3(float s, unsigned (&u)[3]) {
  u[0] = __float_as_uint(s);
  const float r1 = s - __uint_as_float(u[0] & 0xffff0000u);
  u[1] = __float_as_uint(r1);
  u[2] = __float_as_uint(r1 - __uint_as_float(u[1] & 0xffff0000u));
}
// upper halves of (lo, hi) as one word
__device__ __forceinline__ unsigned pack_hi(unsigned lo, unsigned hi) { return __builtin_amdgcn_perm(hi, lo, 0x07060302u); }

typedef unsigned u32x4 __attribute__((ext_vector_type(4)));

// ------------------------------------------------------- biases and cache write
struct WriteArgs {
  void* z;             // [T, ldz]: q | k | v from columns 0, ok, ov, heads padded to dkp / dvp
  long ldz;
  const float* b;      // [nq + nk + nv] biases in that order
  void* pages;
  const int* slots;    // [T], -1: not cached
  int T, nq, G, dkp, dvp, ok, ov;
};

template <typename T>
struct Vec8 {
  T v[8];
};

// One thread: 8 columns of 8 rows. q gets its bias in place; k and v get theirs and
// go to the page, v as 8 tokens of a dim where the rows allow it.
template <typename T>
__global__ __launch_bounds__(256) void write_kv(WriteArgs a) {
  const int nk = a.G * a.dkp, nv = a.G * a.dvp;
  const int col = (blockIdx.x * 256 + threadIdx.x) * 8, r0 = blockIdx.y * 8, nr = min(8, a.T - r0);
  if (col >= a.nq + nk + nv) return;
  const int kind = col < a.nq ? 0 : col < a.nq + nk ? 1 : 2;
  const int c = kind == 0 ? col : kind == 1 ? col - a.nq : col - a.nq - nk;
  const int zc = kind == 0 ? c : kind == 1 ? a.ok + c : a.ov + c;
  float b[8];
#pragma unroll
  for (int i = 0; i < 8; ++i) b[i] = a.b[col + i];
  Vec8<T> x[8];
#pragma unroll
  for (int r = 0; r < 8; ++r) {
    x[r] = *(const Vec8<T>*)((const T*)a.z + (long)(r0 + min(r, nr - 1)) * a.ldz + zc);
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      if constexpr (sizeof(T) == 2) x[r].v[i] = f2bf(bf2f(x[r].v[i]) + b[i]);
      else x[r].v[i] += b[i];
    }
  }
  if (kind == 0) {
#pragma unroll
    for (int r = 0; r < 8; ++r)
      if (r < nr) *(Vec8<T>*)((T*)a.z + (long)(r0 + r) * a.ldz + zc) = x[r];
    return;
  }
  const long per = (long)PAGE * (a.dkp + a.dvp);  // elements of one head's page
  const int g = c / (kind == 1 ? a.dkp : a.dvp), d = c - g * (kind == 1 ? a.dkp : a.dvp);
  int sl[8];
#pragma unroll
  for (int r = 0; r < 8; ++r) sl[r] = r < nr ? a.slots[r0 + r] : -1;
  if (kind == 1) {
#pragma unroll
    for (int r = 0; r < 8; ++r)
      if (sl[r] >= 0)
        *(Vec8<T>*)((T*)a.pages + ((long)(sl[r] / PAGE) * a.G + g) * per + k_at(sl[r] % PAGE, d, a.dkp / 32)) = x[r];
    return;
  }
  bool whole = sl[0] >= 0 && (sl[0] & 7) == 0;
#pragma unroll
  for (int r = 1; r < 8; ++r) whole &= sl[r] == sl[0] + r;
  if (whole) {
    T* p = (T*)a.pages + ((long)(sl[0] / PAGE) * a.G + g) * per + PAGE * a.dkp;
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      Vec8<T> y;
#pragma unroll
      for (int r = 0; r < 8; ++r) y.v[r] = x[r].v[i];
      *(Vec8<T>*)(p + v_at(sl[0] % PAGE, d + i)) = y;
    }
    return;
  }
#pragma unroll
  for (int r = 0; r < 8; ++r) {
    if (sl[r] < 0) continue;
    T* p = (T*)a.pages + ((long)(sl[r] / PAGE) * a.G + g) * per + PAGE * a.dkp;
#pragma unroll
    for (int i = 0; i < 8; ++i) p[v_at(sl[r] % PAGE, d + i)] = x[r].v[i];
  }
}

// ------------------------------------------------------------------------ rows
struct Args {
  const void* q;       // [T, ldq], head h at column h dkp
  long ldq;
  const void* pages;
  void* o;             // [T, ldo], head h at column h dvp
  long ldo;
  const int* bt;       // [sequences, W]
  int W;
  const int* tok_seq;  // per query: its block-table row and its position
  const int* tok_pos;
  const int* rows;     // its batch row, or null: the same
  const int4* items;   // tiles: (first batch row, block-table row, position, queries <= 16)
  float* po;           // partial results of split rows: [row, split][heads][dvp]
  float* pml;          // [row, split][heads][2]
  const float* sc;     // [heads]
  const unsigned short* talk;  // bf16 MFMA fragments (rows: [HT][NC][64][8]; tiles: [MT][64][8])
  const float* talk32; // [heads][heads], the plain kernel's
  const float* bias;   // [nfar + 1][ldb]
  int ldb, nfar;
  int H, G, R, dkp, dvp, nsplit;
};

// Heads 16 ht + .. of one token per MFMA tile. Four waves take pages of the split in
// turn, key heads one after another with the next one's fragments in flight.
template <int HT, int NK, int ND>
__global__ __launch_bounds__(256, 2) void attn_rows(Args a) {
  constexpr int NC = (HT + 1) / 2, NL = 2 * NK > ND ? 2 * NK : ND;
  const int lane = threadIdx.x & 63, w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), n = lane & 15, q = lane >> 4;
  const int row = blockIdx.x / a.nsplit, sp = blockIdx.x - row * a.nsplit;
  const int pos = a.tok_pos[row], npage = pos / PAGE + 1;
  const int per = (npage + a.nsplit - 1) / a.nsplit, p0 = sp * per, p1 = min(npage, p0 + per);
  const int* bt = a.bt + (long)a.tok_seq[row] * a.W;
  const long brow = a.rows ? a.rows[row] : row;
  __shared__ __attribute__((aligned(16))) float lo[4][HT * ND * 256];
  __shared__ float lm[4][HT * 16][2];

  bf16x8 qf[HT][NK];
  float sc[HT][4];
  int grp[HT][4], gcol[HT];  // key head of this lane's S rows and of its mixed column
#pragma unroll
  for (int t = 0; t < HT; ++t) {
    const int h = 16 * t + n;
    const unsigned short* qp = (const unsigned short*)a.q + brow * a.ldq + (long)h * a.dkp + 8 * q;
#pragma unroll
    for (int ks = 0; ks < NK; ++ks) qf[t][ks] = h < a.H ? *(const bf16x8*)(qp + 32 * ks) : bf16x8{};
    gcol[t] = h < a.H ? h / a.R : -1;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int hr = 16 * t + 4 * q + r;
      sc[t][r] = hr < a.H ? a.sc[hr] : 0.f;
      grp[t][r] = hr < a.H ? hr / a.R : -1;
    }
  }
  bf16x8 tf[HT][NC];
#pragma unroll
  for (int t = 0; t < HT; ++t)
#pragma unroll
    for (int c = 0; c < NC; ++c) tf[t][c] = *(const bf16x8*)(a.talk + ((t * NC + c) * 64 + lane) * 8);

  f32x4 acc[HT][ND];
  float m[HT], l[HT], bfar[HT];
  u32x4 pf[HT];
  f32x4 S[HT][2];
#pragma unroll
  for (int t = 0; t < HT; ++t) {
    m[t] = 0.f;
    l[t] = 0.f;
    bfar[t] = 16 * t + n < a.H ? a.bias[(long)a.nfar * a.ldb + 16 * t + n] : 0.f;
#pragma unroll
    for (int d = 0; d < ND; ++d) acc[t][d] = f32x4{};
  }

  const int np = p1 > p0 + w ? (p1 - p0 - w + 3) / 4 : 0;  // this wave's pages
  const int nst = np * 2 * a.G;                            // K then V of every key head
  const long hpage = (long)PAGE * (a.dkp + a.dvp);
  // stage st: page st / 2G, its K of head st % 2G or V of head st % 2G - G
  int lst = 0, lpage = 0;  // the loader's place
  const unsigned short* lbase = nullptr;
  auto load = [&](bf16x8 (&f)[NL]) {
    if (lpage >= np) return;
    if (lst == 0) lbase = (const unsigned short*)a.pages + (long)bt[p0 + w + 4 * lpage] * a.G * hpage + 8 * lane;
    const bool isv = lst >= a.G;
    const unsigned short* p = lbase + (isv ? lst - a.G : lst) * hpage + (isv ? PAGE * a.dkp : 0);
    if (!isv) {
#pragma unroll
      for (int i = 0; i < 2 * NK; ++i) f[i] = __builtin_nontemporal_load((const bf16x8*)(p + 512 * i));
    } else {
#pragma unroll
      for (int i = 0; i < ND; ++i) f[i] = __builtin_nontemporal_load((const bf16x8*)(p + 512 * i));
    }
    if (++lst == 2 * a.G) lst = 0, ++lpage;
  };
  int cst = 0, cpage = 0;  // the consumer's
  auto consume = [&](const bf16x8 (&f)[NL]) {
    if (cst < a.G) {
      const int g = cst, h0 = g * a.R, h1 = h0 + a.R - 1;
#pragma unroll
      for (int t = 0; t < HT; ++t) {
        if (16 * t > h1 || 16 * t + 15 < h0) continue;
#pragma unroll
        for (int kt = 0; kt < 2; ++kt) {
          f32x4 s{};
#pragma unroll
          for (int ks = 0; ks < NK; ++ks) s = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qf[t][ks], f[kt * NK + ks], s, 0, 0, 0);
#pragma unroll
          for (int r = 0; r < 4; ++r) S[t][kt][r] = grp[t][r] == g ? s[r] : S[t][kt][r];
        }
      }
      if (g == a.G - 1) {  // every head's scores of the page are there: mix, softmax
        const int tok0 = (p0 + w + 4 * cpage) * PAGE;
        bf16x8 part[NC][2][3];
#pragma unroll
        for (int c = 0; c < NC; ++c)
#pragma unroll
          for (int kt = 0; kt < 2; ++kt) {
            u32x4 x[3] = {};
#pragma unroll
            for (int hf = 0; hf < 2; ++hf) {
              const int t = 2 * c + hf;
              if (t >= HT) continue;
              unsigned u[4][3];
#pragma unroll
              for (int r = 0; r < 4; ++r) split3(S[t][kt][r] * sc[t][r], u[r]);
#pragma unroll
              for (int j = 0; j < 3; ++j) {
                x[j][2 * hf] = pack_hi(u[0][j], u[1][j]);
                x[j][2 * hf + 1] = pack_hi(u[2][j], u[3][j]);
              }
            }
#pragma unroll
            for (int j = 0; j < 3; ++j) part[c][kt][j] = __builtin_bit_cast(bf16x8, x[j]);
          }
        const bool near = pos - (tok0 + PAGE - 1) < a.nfar, edge = tok0 + PAGE - 1 > pos;
#pragma unroll
        for (int t = 0; t < HT; ++t) {
          f32x4 D[2];
#pragma unroll
          for (int kt = 0; kt < 2; ++kt) {
            D[kt] = f32x4{bfar[t], bfar[t], bfar[t], bfar[t]};
            if (near) {
#pragma unroll
              for (int r = 0; r < 4; ++r) {
                const int dist = min(max(pos - (tok0 + 2 * (4 * q + r) + kt), 0), a.nfar);
                D[kt][r] = a.bias[(long)dist * a.ldb + 16 * t + n];
              }
            }
#pragma unroll
            for (int c = 0; c < NC; ++c)
#pragma unroll
              for (int j = 2; j >= 0; --j)
                D[kt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(part[c][kt][j], tf[t][c], D[kt], 0, 0, 0);
            if (edge) {
#pragma unroll
              for (int r = 0; r < 4; ++r)
                if (tok0 + 2 * (4 * q + r) + kt > pos) D[kt][r] = NEG;
            }
          }
          float mx = m[t];
#pragma unroll
          for (int r = 0; r < 4; ++r) mx = fmaxf(mx, fmaxf(D[0][r], D[1][r]));
          if (__any(mx > m[t] + RESCALE)) {
            mx = xor32_max(xor16_max(mx));
            const float al = __builtin_amdgcn_exp2f(m[t] - mx);
            m[t] = mx;
            l[t] *= al;
#pragma unroll
            for (int d = 0; d < ND; ++d) acc[t][d] *= al;
          }
          float p[2][4];
#pragma unroll
          for (int r = 0; r < 4; ++r)
#pragma unroll
            for (int kt = 0; kt < 2; ++kt) {
              p[kt][r] = __builtin_amdgcn_exp2f(D[kt][r] - m[t]);
              l[t] += p[kt][r];
            }
#pragma unroll
          for (int r = 0; r < 4; ++r) pf[t][r] = pack_bf16x2(p[0][r], p[1][r]);  // tokens 8q + 2r, + 1
        }
      }
    } else {
      const int g = cst - a.G, h0 = g * a.R, h1 = h0 + a.R - 1;
#pragma unroll
      for (int t = 0; t < HT; ++t) {
        if (16 * t > h1 || 16 * t + 15 < h0) continue;
        u32x4 x;
#pragma unroll
        for (int r = 0; r < 4; ++r) x[r] = gcol[t] == g ? pf[t][r] : 0u;
        const bf16x8 pb = __builtin_bit_cast(bf16x8, x);
#pragma unroll
        for (int d = 0; d < ND; ++d) acc[t][d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(f[d], pb, acc[t][d], 0, 0, 0);
      }
    }
    if (++cst == 2 * a.G) cst = 0, ++cpage;
  };
  {
    bf16x8 fa[NL], fb[NL];
#pragma unroll
    for (int t = 0; t < HT; ++t) S[t][0] = S[t][1] = f32x4{}, pf[t] = u32x4{};
    load(fa);
    for (int st = 0; st < nst; st += 2) {  // nst is even
      load(fb);
      consume(fa);
      load(fa);
      consume(fb);
    }
  }
  // lane: O^T[dim 16 d + 4q + r][head 16 t + n]; the four waves' results meet in LDS
#pragma unroll
  for (int t = 0; t < HT; ++t) {
    l[t] = xor32_sum(xor16_sum(l[t]));
    if (q == 0) lm[w][16 * t + n][0] = m[t], lm[w][16 * t + n][1] = l[t];
#pragma unroll
    for (int d = 0; d < ND; ++d) *(f32x4*)(&lo[w][((t * ND + d) * 64 + lane) * 4]) = acc[t][d];
  }
  __syncthreads();
  for (int i = w; i < HT * ND; i += 4) {
    const int t = i / ND, d = i - t * ND, h = 16 * t + n;
    float M = 0.f, L = 0.f;
#pragma unroll
    for (int s = 0; s < 4; ++s) M = fmaxf(M, lm[s][h][0]);
    f32x4 o{};
#pragma unroll
    for (int s = 0; s < 4; ++s) {
      const float f = __builtin_amdgcn_exp2f(lm[s][h][0] - M);
      L += f * lm[s][h][1];
      o += f * *(const f32x4*)(&lo[s][(i * 64 + lane) * 4]);
    }
    if (h >= a.H) continue;
    if (a.nsplit == 1) {
      const float inv = 1.0f / (L + __builtin_amdgcn_exp2f(-M));
      uint2 pk;
      pk.x = pack_bf16x2(o[0] * inv, o[1] * inv);
      pk.y = pack_bf16x2(o[2] * inv, o[3] * inv);
      *(uint2*)((unsigned short*)a.o + brow * a.ldo + (long)h * a.dvp + 16 * d + 4 * q) = pk;
    } else {
      const long pr = ((long)row * a.nsplit + sp) * a.H + h;
      *(f32x4*)(a.po + pr * a.dvp + 16 * d + 4 * q) = o;
      if (d == 0 && q == 0) a.pml[2 * pr] = M, a.pml[2 * pr + 1] = L;
    }
  }
}

// splits of one (row, head): 64 threads, 2 or 1 dims each (dvp 128 or 64)
__global__ __launch_bounds__(64) void merge(Args a) {
  const int row = blockIdx.x / a.H, h = blockIdx.x - row * a.H, e = a.dvp / 64, d = threadIdx.x * e;
  const long pr = (long)row * a.nsplit * a.H + h;
  float M = 0.f;
  for (int s = 0; s < a.nsplit; ++s) M = fmaxf(M, a.pml[2 * (pr + (long)s * a.H)]);
  float L = __builtin_amdgcn_exp2f(-M), o0 = 0.f, o1 = 0.f;
  for (int s = 0; s < a.nsplit; ++s) {
    const long p = pr + (long)s * a.H;
    const float f = __builtin_amdgcn_exp2f(a.pml[2 * p] - M);
    L += f * a.pml[2 * p + 1];
    const float* x = a.po + p * a.dvp + d;
    o0 += f * x[0];
    if (e == 2) o1 += f * x[1];
  }
  const long brow = a.rows ? a.rows[row] : row;
  unsigned short* op = (unsigned short*)a.o + brow * a.ldo + (long)h * a.dvp + d;
  op[0] = f2bf(o0 / L);
  if (e == 2) op[1] = f2bf(o1 / L);
}

// ----------------------------------------------------------------------- tiles
// row i <- element of register i of lane group ..: x[j] of lane group g becomes
// lane group j's x[g]
__device__ __forceinline__ void transpose4(unsigned (&x)[4]) {
  const auto a = __builtin_amdgcn_permlane32_swap(x[0], x[2], false, false);
  const auto b = __builtin_amdgcn_permlane32_swap(x[1], x[3], false, false);
  const auto c = __builtin_amdgcn_permlane16_swap(a[0], b[0], false, false);
  const auto d = __builtin_amdgcn_permlane16_swap(a[1], b[1], false, false);
  x[0] = c[0], x[1] = c[1], x[2] = d[0], x[3] = d[1];
}

// 16 queries of one portion, all heads. Wave w: queries 4w .. 4w + 3. Heads sit in
// slots of 4 that share a key head (slot s: key head s / QPG, its heads
// 4 (s % QPG) .., those past the group's end empty). K and V pages come by LDS-DMA:
// the next K while the scores are mixed, the next V while they are computed.
template <int NS, int NK, int ND>
__global__ __launch_bounds__(256, NS * (NK + ND) > 64 ? 1 : 2) void attn_tiles(Args a) {
  constexpr int MT = (NS + 3) / 4;
  constexpr bool QRES = NS * ND < 64;  // queries stay in registers
  __shared__ __attribute__((aligned(1024))) char smem[NS * (2 * NK + ND + 4) * 1024];
  char* const ks = smem;
  char* const vs = smem + NS * 2 * NK * 1024;
  const int lane = threadIdx.x & 63, w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), n = lane & 15, q = lane >> 4;
  char* const ps = vs + NS * ND * 1024 + w * NS * 1024;  // this wave's P: [slot][16 rows][32 keys]
  const int4 it = a.items[blockIdx.x];
  const int qpg = (a.R + 3) / 4, nslot = a.G * qpg;
  const int* bt = a.bt + (long)it.y * a.W;
  const int npage = (it.z + it.w - 1) / PAGE + 1;
  const long hpage = (long)PAGE * (a.dkp + a.dvp) * 2;  // bytes of one head's page
  const int posw = it.z + 4 * w;                        // position of the wave's first query

  // this lane's query row of the S tiles: query n >> 2, head n & 3 of the slot
  const unsigned short* qrow = (const unsigned short*)a.q + (long)(it.x + min(4 * w + (n >> 2), it.w - 1)) * a.ldq + 8 * q;
  auto load_q = [&](bf16x8 (&f)[NK], int s) {
    const int hr = 4 * (s % qpg) + (n & 3);
    const unsigned short* p = qrow + (long)(s / qpg * a.R + hr) * a.dkp;
#pragma unroll
    for (int k = 0; k < NK; ++k) f[k] = s < nslot && hr < a.R ? *(const bf16x8*)(p + 32 * k) : bf16x8{};
  };
  bf16x8 qf[QRES ? NS : 1][NK];
  if constexpr (QRES) {
#pragma unroll
    for (int s = 0; s < NS; ++s) load_q(qf[s], s);
  }
  float sc[NS][4];  // uniform
#pragma unroll
  for (int s = 0; s < NS; ++s)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int hr = 4 * (s % qpg) + r;
      sc[s][r] = s < nslot && hr < a.R ? a.sc[s / qpg * a.R + hr] : 0.f;
    }
  bf16x8 tf[MT];
  f32x4 bfar[MT];
#pragma unroll
  for (int t = 0; t < MT; ++t) {
    tf[t] = *(const bf16x8*)(a.talk + (t * 64 + lane) * 8);
    bfar[t] = *(const f32x4*)(a.bias + (long)a.nfar * a.ldb + 16 * t + 4 * q);
  }

  // page chunks of 1 KB, dealt to the waves
  auto dma_k = [&](int pg) {
    const char* base = (const char*)a.pages + (long)bt[pg] * a.G * hpage + 16 * lane;
    for (int i = w; i < a.G * 2 * NK; i += 4) glds16(base + (i / (2 * NK)) * hpage + (i % (2 * NK)) * 1024, ks + i * 1024);
  };
  auto dma_v = [&](int pg) {
    const char* base = (const char*)a.pages + (long)bt[pg] * a.G * hpage + PAGE * a.dkp * 2 + 16 * lane;
    for (int i = w; i < a.G * ND; i += 4) glds16(base + (i / ND) * hpage + (i % ND) * 1024, vs + i * 1024);
  };
  auto drain = [&]() {
    asm volatile("s_waitcnt vmcnt(0) lgkmcnt(0)" ::: "memory");
    __syncthreads();
  };

  f32x4 acc[NS][ND];
  f32x4 m[4][MT];  // running maxima of (query, slot 4t + q, head)
  float l[NS];
#pragma unroll
  for (int s = 0; s < NS; ++s) {
    l[s] = 0.f;
#pragma unroll
    for (int d = 0; d < ND; ++d) acc[s][d] = f32x4{};
  }
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int t = 0; t < MT; ++t) m[i][t] = f32x4{};

  dma_k(0);
  drain();
  for (int pg = 0; pg < npage; ++pg) {
    const int tok0 = pg * PAGE;
    if constexpr (QRES) dma_v(pg);
    f32x4 S[NS][2];
#pragma unroll
    for (int s = 0; s < NS; ++s) {
      S[s][0] = S[s][1] = f32x4{};
      if (s < nslot) {
        if constexpr (!QRES) load_q(qf[0], s);
        const char* kp = ks + (s / qpg) * (2 * NK * 1024) + 16 * lane;
#pragma unroll
        for (int kt = 0; kt < 2; ++kt)
#pragma unroll
          for (int k = 0; k < NK; ++k)
            S[s][kt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qf[QRES ? s : 0][k], *(const bf16x8*)(kp + (kt * NK + k) * 1024),
                                                               S[s][kt], 0, 0, 0);
      }
    }
    if constexpr (!QRES) dma_v(pg);
    // K of this page is done with everywhere, V of it is there
    drain();
    if (pg + 1 < npage) dma_k(pg + 1);

    const bool near = posw - (tok0 + PAGE - 1) < a.nfar, edge = tok0 + PAGE - 1 > posw;
    float p0[4][MT][4];
#pragma unroll
    for (int kt = 0; kt < 2; ++kt) {
      unsigned x[3][2][2][4];  // [part][half][head pair][slot of the half, then query]
#pragma unroll
      for (int s = 0; s < 4 * MT; ++s) {
        unsigned u[4][3];
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          if (s < NS) split3(S[s < NS ? s : 0][kt][r] * sc[s < NS ? s : 0][r], u[r]);
          else u[r][0] = u[r][1] = u[r][2] = 0;
        }
#pragma unroll
        for (int j = 0; j < 3; ++j) {
          x[j][s >> 2][0][s & 3] = pack_hi(u[0][j], u[1][j]);
          x[j][s >> 2][1][s & 3] = pack_hi(u[2][j], u[3][j]);
        }
      }
#pragma unroll
      for (int j = 0; j < 3; ++j)
#pragma unroll
        for (int hf = 0; hf < MT; ++hf) transpose4(x[j][hf][0]), transpose4(x[j][hf][1]);
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        f32x4 D[MT];
#pragma unroll
        for (int t = 0; t < MT; ++t) D[t] = bfar[t];
        const int dist = posw + i - (tok0 + 2 * n + kt);
        if (near) {
          const float* bp = a.bias + (long)min(max(dist, 0), a.nfar) * a.ldb + 4 * q;
#pragma unroll
          for (int t = 0; t < MT; ++t) D[t] = *(const f32x4*)(bp + 16 * t);
        }
#pragma unroll
        for (int j = 2; j >= 0; --j) {
          const u32x4 b = {x[j][0][0][i], x[j][0][1][i], MT > 1 ? x[j][MT - 1][0][i] : 0u, MT > 1 ? x[j][MT - 1][1][i] : 0u};
#pragma unroll
          for (int t = 0; t < MT; ++t)
            D[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(tf[t], __builtin_bit_cast(bf16x8, b), D[t], 0, 0, 0);
        }
        // lane: key 2n + kt, slot 4t + q, head r
        float over = -1.f;
#pragma unroll
        for (int t = 0; t < MT; ++t)
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            if (edge && dist < 0) D[t][r] = NEG;
            D[t][r] -= m[i][t][r];
            over = fmaxf(over, D[t][r]);
          }
        if (__any(over > RESCALE)) {
          // new maxima over the 16 keys; sel: the factor of head n & 3, for the lanes that hold its row
          float sel[MT];
#pragma unroll
          for (int t = 0; t < MT; ++t)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
              float up = fmaxf(D[t][r], 0.f);
#pragma unroll
              for (int b = 1; b < 16; b <<= 1) up = fmaxf(up, __shfl_xor(up, b, 16));
              const float f = __builtin_amdgcn_exp2f(-up);
              m[i][t][r] += up;
              D[t][r] -= up;
              if (kt == 1) p0[i][t][r] *= f;
              sel[t] = r == 0 || (n & 3) == r ? f : sel[t];
            }
#pragma unroll
          for (int s = 0; s < NS; ++s) {
            const float g = __shfl(sel[s >> 2], 16 * (s & 3) + (n & 3), 64), f = (n >> 2) == i ? g : 1.f;
            l[s] *= f;
#pragma unroll
            for (int d = 0; d < ND; ++d) acc[s][d] *= f;
          }
        }
#pragma unroll
        for (int t = 0; t < MT; ++t)
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            const float p = __builtin_amdgcn_exp2f(D[t][r]);
            if (kt == 0) p0[i][t][r] = p;
            else if (4 * t + q < NS) {
              // P row 4i + r of slot 4t + q; rows permuted by the slot and 16-B chunks by the row: no bank twice
              const int s = 4 * t + q, rw = 4 * i + r;
              *(unsigned*)(ps + s * 1024 + ((rw ^ (s & 3)) * 64) + (((n >> 2) ^ ((rw >> 2) & 3)) * 16) + (n & 3) * 4) =
                  pack_bf16x2(p0[i][t][r], p);
            }
          }
      }
    }
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    __builtin_amdgcn_wave_barrier();
#pragma unroll
    for (int s = 0; s < NS; ++s) {
      if (s >= nslot) continue;
      const u32x4 pw = *(const u32x4*)(ps + s * 1024 + ((n ^ (s & 3)) * 64) + ((q ^ ((n >> 2) & 3)) * 16));
#pragma unroll
      for (int e = 0; e < 4; ++e) l[s] += __uint_as_float(pw[e] << 16) + __uint_as_float(pw[e] & 0xffff0000u);
      const bf16x8 pb = __builtin_bit_cast(bf16x8, pw);
      const char* vp = vs + (s / qpg) * (ND * 1024) + 16 * lane;
#pragma unroll
      for (int d = 0; d < ND; ++d)
        acc[s][d] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*(const bf16x8*)(vp + d * 1024), pb, acc[s][d], 0, 0, 0);
    }
    drain();  // V is done with everywhere, the next K is there
  }

  // rows' maxima to the lanes that hold the rows: [slot][row]
  float* mm = (float*)ps;
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int t = 0; t < MT; ++t)
      if (n == 0 && 4 * t + q < NS) *(f32x4*)(mm + (4 * t + q) * 16 + 4 * i) = m[i][t];
  asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
  __builtin_amdgcn_wave_barrier();
  const int qi = 4 * w + (n >> 2);
#pragma unroll
  for (int s = 0; s < NS; ++s) {
    const int hr = 4 * (s % qpg) + (n & 3);
    const float L = xor32_sum(xor16_sum(l[s])) + __builtin_amdgcn_exp2f(-mm[s * 16 + n]);
    if (s >= nslot || hr >= a.R || qi >= it.w) continue;
    const float inv = 1.0f / L;
    unsigned short* op = (unsigned short*)a.o + (long)(it.x + qi) * a.ldo + (long)(s / qpg * a.R + hr) * a.dvp + 4 * q;
#pragma unroll
    for (int d = 0; d < ND; ++d) {
      uint2 pk;
      pk.x = pack_bf16x2(acc[s][d][0] * inv, acc[s][d][1] * inv);
      pk.y = pack_bf16x2(acc[s][d][2] * inv, acc[s][d][3] * inv);
      *(uint2*)(op + 16 * d) = pk;
    }
  }
}

// ----------------------------------------------------------------------- plain
// Any sizes, fp32 or bf16, no MFMA: one workgroup per query token, 64 keys at a time.
// LDS: q [H][dkp], S and mixed S [H][64], O [H][dvp], m, l, alpha [H].
template <typename T>
__device__ __forceinline__ float ld(const T* p) {
  if constexpr (sizeof(T) == 2) return bf2f(*p);
  else return *p;
}

template <typename T>
__global__ __launch_bounds__(256) void attn_plain(Args a) {
  extern __shared__ float lds[];
  const int row = blockIdx.x, tid = threadIdx.x, j = tid & 63, w = tid >> 6;
  const int pos = a.tok_pos[row];
  const int* bt = a.bt + (long)a.tok_seq[row] * a.W;
  const long brow = a.rows ? a.rows[row] : row;
  float* qs = lds;
  float* S = qs + a.H * a.dkp;
  float* P = S + a.H * 64;
  float* O = P + a.H * 64;
  float* m = O + a.H * a.dvp;
  float* l = m + a.H;
  float* al = l + a.H;
  for (int i = tid; i < a.H * a.dkp; i += 256) qs[i] = ld((const T*)a.q + brow * a.ldq + i);
  for (int i = tid; i < a.H * a.dvp; i += 256) O[i] = 0.f;
  for (int i = tid; i < a.H; i += 256) m[i] = 0.f, l[i] = 0.f;
  __syncthreads();
  const long per = (long)PAGE * (a.dkp + a.dvp);
  for (int k0 = 0; k0 <= pos; k0 += 64) {
    const int key = k0 + j;
    const bool ok = key <= pos;
    const T* pg = (const T*)a.pages + (ok ? (long)bt[key / PAGE] * a.G * per : 0);
    for (int h = w; h < a.H; h += 4) {
      float s = 0.f;
      if (ok) {
        const T* kp = pg + (h / a.R) * per;
        for (int d = 0; d < a.dkp; ++d) s = __builtin_fmaf(qs[h * a.dkp + d], ld(kp + k_at(key % PAGE, d, a.dkp / 32)), s);
      }
      S[h * 64 + j] = s * a.sc[h];
    }
    __syncthreads();
    for (int h = w; h < a.H; h += 4) {
      float s = a.bias[(long)min(max(pos - key, 0), a.nfar) * a.ldb + h];
      for (int g = 0; g < a.H; ++g) s = __builtin_fmaf(a.talk32[h * a.H + g], S[g * 64 + j], s);
      if (!ok) s = NEG;
      float mx = s;
#pragma unroll
      for (int b = 1; b < 64; b <<= 1) mx = fmaxf(mx, __shfl_xor(mx, b, 64));
      const float mo = m[h], mn = fmaxf(mo, mx), p = exp2f(s - mn), ps = wave_sum(p);
      P[h * 64 + j] = p;
      if (j == 0) {
        const float f = exp2f(mo - mn);
        al[h] = f;
        m[h] = mn;
        l[h] = l[h] * f + ps;
      }
    }
    __syncthreads();
    const int nk = min(64, pos + 1 - k0);
    for (int i = tid; i < a.H * a.dvp; i += 256) {
      const int h = i / a.dvp, d = i - h * a.dvp;
      float o = O[i] * al[h];
      for (int t = 0; t < nk; ++t) {
        const T* vp = (const T*)a.pages + ((long)bt[(k0 + t) / PAGE] * a.G + h / a.R) * per + PAGE * a.dkp;
        o = __builtin_fmaf(P[h * 64 + t], ld(vp + v_at((k0 + t) % PAGE, d)), o);
      }
      O[i] = o;
    }
    __syncthreads();
  }
  for (int i = tid; i < a.H * a.dvp; i += 256) {
    const int h = i / a.dvp;
    const float y = O[i] / (l[h] + exp2f(-m[h]));
    if constexpr (sizeof(T) == 2) ((T*)a.o)[brow * a.ldo + i] = f2bf(y);
    else ((T*)a.o)[brow * a.ldo + i] = y;
  }
}

template <int HT, int NK, int ND>
void run_rows(const Args& a, int nrows, hipStream_t s) {
  hipLaunchKernelGGL((attn_rows<HT, NK, ND>), dim3((unsigned)(nrows * a.nsplit)), dim3(256), 0, s, a);
  if (a.nsplit > 1) hipLaunchKernelGGL(merge, dim3((unsigned)(nrows * a.H)), dim3(64), 0, s, a);
}
template <int NK, int ND>
void rows_ht(const Args& a, int nrows, hipStream_t s) {
  if (a.H <= 16) run_rows<1, NK, ND>(a, nrows, s);
  else if (a.H <= 32) run_rows<2, NK, ND>(a, nrows, s);
  else run_rows<4, NK, ND>(a, nrows, s);
}
template <int NK, int ND>
void tiles_ns(const Args& a, int nitems, int nslot, hipStream_t s) {
  const dim3 grid((unsigned)nitems), block(256);
  if (nslot <= 2) hipLaunchKernelGGL((attn_tiles<2, NK, ND>), grid, block, 0, s, a);
  else if (nslot <= 4) hipLaunchKernelGGL((attn_tiles<4, NK, ND>), grid, block, 0, s, a);
  else hipLaunchKernelGGL((attn_tiles<8, NK, ND>), grid, block, 0, s, a);
}

int check(const Args& a, int n) {
  if (n <= 0 || a.H <= 0 || a.G <= 0 || a.H % a.G || a.dkp <= 0 || a.dvp <= 0 || a.dkp % 32 || a.dvp % 16 || a.W <= 0 ||
      a.nfar < 0 || a.ldq < (long)a.H * a.dkp || a.ldo < (long)a.H * a.dvp || a.ldb < a.H)
    return KGS_ERR_SHAPE;
  if (a.ldq % 8 || a.ldo % 8 || a.ldb % 4 || (((uintptr_t)a.q | (uintptr_t)a.o | (uintptr_t)a.pages | (uintptr_t)a.bias) & 15))
    return KGS_ERR_ALIGN;
  return KGS_OK;
}

}  // namespace talking
}  // namespace kgs

// z [T, ldz] holds q from column 0, k from ok, v from ov (heads padded to dkp / dvp);
// b their biases one after another (nq + G dkp + G dvp). q += b in place, k + b and
// v + b go to their slots.
KGS_EXPORT int kgs_talking_write(void* z, long ldz, const void* b, void* pages, const void* slots, int T, int nq, int G,
                                 int dkp, int dvp, int ok, int ov, int f32, hipStream_t s) {
  using namespace kgs::talking;
  if (T <= 0 || nq <= 0 || G <= 0 || dkp <= 0 || dvp <= 0 || dkp % 32 || dvp % 16 || nq % 8 || ok < nq ||
      ldz < ok + G * dkp || ldz < ov + G * dvp || T > 8 * 65535)
    return KGS_ERR_SHAPE;
  if (ldz % 8 || ok % 8 || ov % 8 || (((uintptr_t)z | (uintptr_t)pages) & 15)) return KGS_ERR_ALIGN;
  WriteArgs a{z, ldz, (const float*)b, pages, (const int*)slots, T, nq, G, dkp, dvp, ok, ov};
  const dim3 grid(((nq + G * (dkp + dvp)) / 8 + 255) / 256, (T + 7) / 8);
  if (f32) hipLaunchKernelGGL(write_kv<float>, grid, dim3(256), 0, s, a);
  else hipLaunchKernelGGL(write_kv<unsigned short>, grid, dim3(256), 0, s, a);
  return (int)hipGetLastError();
}

// nrows query tokens, each over its sequence's pages up to its position. bf16 with
// dkp, dvp 64 or 128 and at most 64 heads; plain != 0 (or fp32): any sizes.
KGS_EXPORT int kgs_talking_rows(const void* q, long ldq, const void* pages, void* o, long ldo, const void* bt, int W,
                                const void* tok_seq, const void* tok_pos, const void* rows, void* po, void* pml,
                                const void* sc, const void* talk, const void* bias, int ldb, int nfar, int nrows, int H,
                                int G, int dkp, int dvp, int nsplit, int plain, int f32, hipStream_t s) {
  using namespace kgs::talking;
  Args a{q, ldq, pages, o, ldo, (const int*)bt, W, (const int*)tok_seq, (const int*)tok_pos, (const int*)rows, nullptr,
         (float*)po, (float*)pml, (const float*)sc, (const unsigned short*)talk, (const float*)talk, (const float*)bias,
         ldb, nfar, H, G, G ? H / G : 0, dkp, dvp, nsplit};
  if (int rc = check(a, nrows)) return rc;
  if (plain || f32) {
    const size_t lds = ((size_t)H * (dkp + dvp + 128 + 3)) * 4;
    if (lds > 160 * 1024) return KGS_ERR_SHAPE;
    const void* fn = f32 ? (const void*)attn_plain<float> : (const void*)attn_plain<unsigned short>;
    if (lds > 64 * 1024) {
      const hipError_t e = hipFuncSetAttribute(fn, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
      if (e != hipSuccess) return (int)e;
    }
    if (f32) hipLaunchKernelGGL(attn_plain<float>, dim3(nrows), dim3(256), lds, s, a);
    else hipLaunchKernelGGL(attn_plain<unsigned short>, dim3(nrows), dim3(256), lds, s, a);
    return (int)hipGetLastError();
  }
  if (H > 64 || (dkp != 64 && dkp != 128) || (dvp != 64 && dvp != 128)) return KGS_ERR_ARG;
  if (nsplit <= 0 || (nsplit > 1 && (!po || !pml)) || (long)nrows * nsplit > 0x7fffffff || (long)nrows * H > 0x7fffffff)
    return KGS_ERR_SHAPE;
  if (dkp == 64) dvp == 64 ? rows_ht<2, 4>(a, nrows, s) : rows_ht<2, 8>(a, nrows, s);
  else dvp == 64 ? rows_ht<4, 4>(a, nrows, s) : rows_ht<4, 8>(a, nrows, s);
  return (int)hipGetLastError();
}

// Prompt portions: nitems blocks of up to 16 consecutive queries (first batch row,
// block-table row, first position, queries). bf16, dkp and dvp 64 or 128, at most 8 slots
// of 4 heads (G ceil(H / G / 4)); talk and bias in slot order, ldb = 16 ceil(slots / 4).
KGS_EXPORT int kgs_talking_tiles(const void* q, long ldq, const void* pages, void* o, long ldo, const void* bt, int W,
                                 const void* items, int nitems, const void* sc, const void* talk, const void* bias,
                                 int ldb, int nfar, int H, int G, int dkp, int dvp, hipStream_t s) {
  using namespace kgs::talking;
  Args a{};
  a.q = q, a.ldq = ldq, a.pages = pages, a.o = o, a.ldo = ldo, a.bt = (const int*)bt, a.W = W;
  a.items = (const int4*)items, a.sc = (const float*)sc, a.talk = (const unsigned short*)talk;
  a.bias = (const float*)bias, a.ldb = ldb, a.nfar = nfar, a.H = H, a.G = G, a.R = G ? H / G : 0;
  a.dkp = dkp, a.dvp = dvp, a.nsplit = 1;
  if (int rc = check(a, nitems)) return rc;
  const int nslot = G * ((H / G + 3) / 4);
  if (nslot > 8 || (dkp != 64 && dkp != 128) || (dvp != 64 && dvp != 128)) return KGS_ERR_ARG;
  if (ldb < (nslot + 3) / 4 * 16 || ((uintptr_t)items & 15)) return KGS_ERR_SHAPE;
  if (dkp == 64) dvp == 64 ? tiles_ns<2, 4>(a, nitems, nslot, s) : tiles_ns<2, 8>(a, nitems, nslot, s);
  else dvp == 64 ? tiles_ns<4, 4>(a, nitems, nslot, s) : tiles_ns<4, 8>(a, nitems, nslot, s);
  return (int)hipGetLastError();
}
