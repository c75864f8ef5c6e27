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
// The mixture is an MFMA over heads whose products are exact: talk is a bf16 number
// that fp16 holds (to 2^-25 where it is below 2^-14), and a score enters as two fp16 parts
// that hold 22 of its bits, or 2^-24: less than the fp32 sum of the score itself
// loses (beyond fp16's range a part saturates). What makes it cheap is that no score
// leaves the registers for it:
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
#include <type_traits>

#include "acc_regs.h"
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

// two fp16 parts of two fp32 values: parts truncated, so a value out of range saturates
typedef _Float16 f16x2 __attribute__((ext_vector_type(2)));
typedef _Float16 f16x8 __attribute__((ext_vector_type(8)));
__device__ __forceinline__ void split2(float a, float b, unsigned& hi, unsigned& lo) {
  const f16x2 h = __builtin_bit_cast(f16x2, __builtin_amdgcn_cvt_pkrtz(a, b));
  // one v_fma_mix_f32 each
  const float ra = __builtin_fmaf((float)h[0], -1.0f, a), rb = __builtin_fmaf((float)h[1], -1.0f, b);
  hi = __builtin_bit_cast(unsigned, h);
  lo = __builtin_bit_cast(unsigned, __builtin_amdgcn_cvt_pkrtz(ra, rb));
}

typedef unsigned u32x4 __attribute__((ext_vector_type(4)));
typedef __bf16 bf16x2 __attribute__((ext_vector_type(2)));

// ------------------------------------------------------- biases and cache write
struct WriteArgs {
  void* z;             // [T, ldz]: q | k | v from columns 0, ok, ov, heads padded to dkp / dvp
  long ldz;
  const float* b;      // [nq + nk + nv] biases in that order, or null
  void* pages;
  const int* slots;    // [T], -1: not cached
  int T, nq, G, dkp, dvp, ok, ov;
  // rotary positions of q and k, neighbouring dims paired: [npos][rot] (cos, sin) of the
  // pairs of the first `rot` dims (a multiple of 8), or null
  const float* cs;
  const int* pos;      // [T]
  int npos, rot;
  // RMS norm of q and k per `seg` columns (`dim` of them without the padding) times wq / wk [seg]
  const float *wq, *wk;
  int seg, dim;
  float eps;
  // q at position p times 1 + coef ln(floor((p + 1) / every) + 1); every 0: none
  float coef;
  int every;
};

template <typename T>
struct Vec8 {
  T v[8];
};

// One thread: 8 columns of 8 rows. q gets its bias (norm, rotation, temperature) in place; k and v
// get theirs and go to the page, v as 8 tokens of a dim where the rows allow it. NORM: lanes of a
// norm's columns: 0 no norm, 8 or 16, 1 any number (workgroups of whole norms, sums through LDS).
template <typename T, int NORM>
__global__ __launch_bounds__(256) void write_kv(WriteArgs a) {
  const int nk = a.G * a.dkp, nv = a.G * a.dvp;
  const int per_wg = NORM == 1 ? 256 / (a.seg / 8) * (a.seg / 8) : 256;
  const int col = (blockIdx.x * per_wg + threadIdx.x) * 8, r0 = blockIdx.y * 8, nr = min(8, a.T - r0);
  const bool in = col < a.nq + nk + nv && (int)threadIdx.x < per_wg;
  if (NORM != 1 && !in) return;
  const int kind = !in || col >= a.nq + nk ? 2 : col < a.nq ? 0 : 1;
  const int c = !in ? 0 : kind == 0 ? col : kind == 1 ? col - a.nq : col - a.nq - nk;
  const int zc = kind == 0 ? c : kind == 1 ? a.ok + c : a.ov + c;
  float b[8] = {}, nw[8];
  if (a.b && in) {
    const f32x4 b0 = *(const f32x4*)(a.b + col), b1 = *(const f32x4*)(a.b + col + 4);
#pragma unroll
    for (int i = 0; i < 4; ++i) b[i] = b0[i], b[4 + i] = b1[i];
  }
  const int dd = kind == 2 ? 0 : c % a.seg;
  const bool turn = a.cs && kind != 2 && dd < a.rot;
  if (NORM && kind != 2) {
    const float* wp = (kind ? a.wk : a.wq) + dd;
#pragma unroll
    for (int i = 0; i < 8; ++i) nw[i] = wp[i];
  }
  int sl[8];
#pragma unroll
  for (int r = 0; r < 8; ++r) sl[r] = r < nr ? a.slots[r0 + r] : -1;
  Vec8<T> x[8];
  auto biased = [&](int r, float (&y)[8]) {
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      if constexpr (sizeof(T) == 2) y[i] = bf2f(x[r].v[i]) + b[i];
      else y[i] = x[r].v[i] + b[i];
    }
  };
#pragma unroll
  for (int r = 0; r < 8; ++r) x[r] = *(const Vec8<T>*)((const T*)a.z + (long)(r0 + min(r, nr - 1)) * a.ldz + zc);
  float inv[8];
  if constexpr (NORM != 0) {
#pragma unroll
    for (int r = 0; r < 8; ++r) {
      float y[8], ss = 0.f;
      biased(r, y);
#pragma unroll
      for (int i = 0; i < 8; ++i) ss = __builtin_fmaf(y[i], y[i], ss);
      if constexpr (NORM != 1) ss = sum8(ss);
      if constexpr (NORM == 16) ss += dpp_move<0x140>(ss);
      inv[r] = ss;
    }
    if constexpr (NORM == 1) {
      __shared__ float part[8][256];
#pragma unroll
      for (int r = 0; r < 8; ++r) part[r][threadIdx.x] = inv[r];
      __syncthreads();
      if (!in) return;
      const int t0 = threadIdx.x - threadIdx.x % (a.seg / 8);
#pragma unroll
      for (int r = 0; r < 8; ++r) {
        inv[r] = 0.f;
        for (int i = 0; i < a.seg / 8; ++i) inv[r] += part[r][t0 + i];
      }
    }
#pragma unroll
    for (int r = 0; r < 8; ++r) inv[r] = 1.0f / sqrtf(inv[r] / a.dim + a.eps);
  }
#pragma unroll
  for (int r = 0; r < 8; ++r) {
    float y[8];
    biased(r, y);
    if (NORM && kind != 2) {
#pragma unroll
      for (int i = 0; i < 8; ++i) y[i] *= inv[r] * nw[i];
    }
    if (turn) {
      const float* p = a.cs + (long)min(max(a.pos[r0 + min(r, nr - 1)], 0), a.npos - 1) * a.rot + dd;
      const f32x4 p0 = *(const f32x4*)p, p1 = *(const f32x4*)(p + 4);
      const float cs[8] = {p0[0], p0[1], p0[2], p0[3], p1[0], p1[1], p1[2], p1[3]};
#pragma unroll
      for (int i = 0; i < 8; i += 2) {
        const float u = y[i], v = y[i + 1];
        y[i] = rope_lo(u, v, cs[i], cs[i + 1]);
        y[i + 1] = rope_hi(u, v, cs[i], cs[i + 1]);
      }
    }
    if (a.every && kind == 0) {
      const float f = __builtin_fmaf(a.coef, logf((float)((a.pos[r0 + min(r, nr - 1)] + 1) / a.every + 1)), 1.0f);
#pragma unroll
      for (int i = 0; i < 8; ++i) y[i] *= f;
    }
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      if constexpr (sizeof(T) == 2) x[r].v[i] = f2bf(y[i]);
      else x[r].v[i] = y[i];
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
  const int4* items;   // tiles, two each: (first batch row, block-table row, position, queries),
                       // (first page, end, partial result or -1, 0)
  const int4* merges;  // split tiles
  int tile;            // queries of a tile
  void* qs;            // tiles: the queries of a workgroup again, in operand order
  float* po;           // partial results of split rows: [row, split][heads][dvp]
  float* pml;          // [row, split][heads][2]
  const float* sc;     // [heads]
  const unsigned short* talk;  // fp16 MFMA fragments (rows: [HT][NC][64][8]; tiles: [MT][64][8])
  const float* talk32; // [heads][heads], the plain kernel's
  const float* bias;   // [nfar + 1][ldb] (tiles: less the last row)
  const float* bfar;   // tiles: the last row
  int ldb, nfar;
  int H, G, R, dkp, dvp, nsplit;
};

// Heads 16 ht + .. of one token per MFMA tile. Four waves take pages of the split in
// turn, key heads one after another with the next one's fragments in flight.
template <int HT, int NK, int ND>
__global__ __launch_bounds__(256, HT > 2 ? 1 : 2) void attn_rows(Args a) {
  constexpr int NC = (HT + 1) / 2, NL = 2 * NK > ND ? 2 * NK : ND;
  const int lane = threadIdx.x & 63, w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), n = lane & 15, q = lane >> 4;
  const int row = blockIdx.x / a.nsplit, sp = blockIdx.x - row * a.nsplit;
  const int pos = a.tok_pos[row], npage = pos / PAGE + 1;
  const int per = (npage + a.nsplit - 1) / a.nsplit, p0 = sp * per, p1 = min(npage, p0 + per);
  const int* bt = a.bt + (long)a.tok_seq[row] * a.W;
  const long brow = a.rows ? a.rows[row] : row;
  __shared__ __attribute__((aligned(16))) float lo[4][HT * ND * 256];
  __shared__ float lm[4][HT * 16][2];
  __shared__ __attribute__((aligned(16))) unsigned short lq[HT * NK * 512];  // the query in operand order

  float sc[HT][4];
  int grp[HT][4], gcol[HT];  // key head of this lane's S rows and of its mixed column
#pragma unroll
  for (int t = 0; t < HT; ++t) {
    const int h = 16 * t + n;
    if ((t & 3) == w || HT < 4) {
      const unsigned short* qp = (const unsigned short*)a.q + brow * a.ldq + (long)h * a.dkp + 8 * q;
#pragma unroll
      for (int ks = 0; ks < NK; ++ks)
        if (HT >= 4 || ((t * NK + ks) & 3) == w)
          *(bf16x8*)(lq + (t * NK + ks) * 512 + 8 * lane) = h < a.H ? *(const bf16x8*)(qp + 32 * ks) : bf16x8{};
    }
    gcol[t] = h < a.H ? h / a.R : -1;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int hr = 16 * t + 4 * q + r;
      sc[t][r] = hr < a.H ? a.sc[hr] : 0.f;
      grp[t][r] = hr < a.H ? hr / a.R : -1;
    }
  }
  f16x8 tf[HT][NC];
#pragma unroll
  for (int t = 0; t < HT; ++t)
#pragma unroll
    for (int c = 0; c < NC; ++c) tf[t][c] = *(const f16x8*)(a.talk + ((t * NC + c) * 64 + lane) * 8);

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
        bf16x8 qf[NK];
#pragma unroll
        for (int ks = 0; ks < NK; ++ks) qf[ks] = *(const bf16x8*)(lq + (t * NK + ks) * 512 + 8 * lane);
#pragma unroll
        for (int kt = 0; kt < 2; ++kt) {
          f32x4 s{};
#pragma unroll
          for (int ks = 0; ks < NK; ++ks) s = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qf[ks], f[kt * NK + ks], s, 0, 0, 0);
#pragma unroll
          for (int r = 0; r < 4; ++r) S[t][kt][r] = grp[t][r] == g ? s[r] : S[t][kt][r];
        }
      }
      if (g == a.G - 1) {  // every head's scores of the page are there: mix, softmax
        const int tok0 = (p0 + w + 4 * cpage) * PAGE;
        f16x8 part[NC][2][2];
#pragma unroll
        for (int c = 0; c < NC; ++c)
#pragma unroll
          for (int kt = 0; kt < 2; ++kt) {
            u32x4 x[2] = {};
#pragma unroll
            for (int hf = 0; hf < 2; ++hf) {
              const int t = 2 * c + hf;
              if (t >= HT) continue;
#pragma unroll
              for (int r = 0; r < 2; ++r) {
                unsigned hi, lo;
                split2(S[t][kt][2 * r] * sc[t][2 * r], S[t][kt][2 * r + 1] * sc[t][2 * r + 1], hi, lo);
                x[0][2 * hf + r] = hi;
                x[1][2 * hf + r] = lo;
              }
            }
            part[c][kt][0] = __builtin_bit_cast(f16x8, x[0]);
            part[c][kt][1] = __builtin_bit_cast(f16x8, x[1]);
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
              for (int j = 1; j >= 0; --j)
                D[kt] = __builtin_amdgcn_mfma_f32_16x16x32_f16(part[c][kt][j], tf[t][c], D[kt], 0, 0, 0);
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
    __syncthreads();
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

// splits (at most 64) of one (row, head): a wave, 2 or 1 dims a lane (dvp 128 or 64).
// TILES: rows are the queries of split tiles, merges = (first batch row, queries, first
// part, parts) of a tile; a part holds `tile` rows.
template <bool TILES>
__global__ __launch_bounds__(TILES ? 256 : 64) void merge(Args a) {
  const int unit = TILES ? 4 * blockIdx.x + __builtin_amdgcn_readfirstlane(threadIdx.x >> 6) : blockIdx.x;
  const int row = unit / a.H, h = unit - row * a.H, e = a.dvp / 64, lane = threadIdx.x & 63;
  long pr = (long)row * a.nsplit * a.H + h, brow, between = a.H;
  int nsplit = a.nsplit;
  if constexpr (TILES) {
    const int4 mt = a.merges[row / a.tile];
    const int q = row % a.tile;
    if (q >= mt.y) return;
    brow = mt.x + q;
    pr = ((long)mt.z * a.tile + q) * a.H + h;
    between = (long)a.tile * a.H;
    nsplit = mt.w;
  } else brow = a.rows ? a.rows[row] : row;
  const float* x = a.po + pr * a.dvp + lane * e;
  const long step = between * a.dvp;
  constexpr int CH = TILES ? 4 : 8;  // splits' loads at a time, the first ahead of the sums
  float2 v[CH];
  auto load = [&](int s0) {
#pragma unroll
    for (int j = 0; j < CH; ++j) {
      const float* p = x + min(s0 + j, nsplit - 1) * step;
      v[j] = e == 2 ? *(const float2*)p : make_float2(*p, 0.f);
    }
  };
  load(0);
  float m = 0.f, l = 0.f;
  if (lane < nsplit) m = a.pml[2 * (pr + lane * between)], l = a.pml[2 * (pr + lane * between) + 1];
  float M = m;
#pragma unroll
  for (int b = 1; b < 64; b <<= 1) M = fmaxf(M, __shfl_xor(M, b, 64));
  const float f = __builtin_amdgcn_exp2f(m - M);
  const float inv = 1.0f / (wave_sum(f * l) + __builtin_amdgcn_exp2f(-M));
  float o0 = 0.f, o1 = 0.f;
  for (int s0 = 0; s0 < nsplit; s0 += CH) {
    if (s0) load(s0);
#pragma unroll
    for (int j = 0; j < CH; ++j) {
      const float g = s0 + j < nsplit ? __shfl(f, s0 + j, 64) : 0.f;
      o0 += g * v[j].x;
      o1 += g * v[j].y;
    }
  }
  unsigned short* op = (unsigned short*)a.o + brow * a.ldo + (long)h * a.dvp + lane * e;
  op[0] = f2bf(o0 * inv);
  if (e == 2) op[1] = f2bf(o1 * inv);
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

// Compile-time loop: f(std::integral_constant<int, i>) for i in [B, E).
template <int B, int E, class F>
__device__ __forceinline__ void static_for(F&& f) {
  if constexpr (B < E) {
    f(std::integral_constant<int, B>{});
    static_for<B + 1, E>(f);
  }
}

// 1 KB of buffer `base` (16 bytes per lane from byte so + vo on) to LDS
__device__ __forceinline__ void dma_chunk(const char* base, int bytes, char* dst, int vo, int so) {
  const __amdgpu_buffer_rsrc_t r = __builtin_amdgcn_make_buffer_rsrc((void*)base, 0, bytes, 0x00020000);
  __builtin_amdgcn_raw_ptr_buffer_load_lds(r, (KGS_LDS void*)dst, 16, vo, so, 0, 0);
}

// ... or to a register
__device__ __forceinline__ bf16x8 load_frag(const char* base, int bytes, int vo, int so) {
  const __amdgpu_buffer_rsrc_t r = __builtin_amdgcn_make_buffer_rsrc((void*)base, 0, bytes, 0x00020000);
  return __builtin_bit_cast(bf16x8, __builtin_amdgcn_raw_buffer_load_b128(r, vo, so, 0));
}

__device__ __forceinline__ void fence() { __builtin_amdgcn_sched_barrier(0); }
// every wave's LDS accesses are done and all but its last VM loads have landed (63: no wait for any)
template <int VM>
__device__ __forceinline__ void bar() {
  fence();
  asm volatile("" ::: "memory");
  __builtin_amdgcn_s_waitcnt(0x0070 | (VM & 15) | ((VM >> 4) << 14));  // vmcnt(VM) lgkmcnt(0)
  asm volatile("s_barrier" ::: "memory");
  fence();
}

// 4 NW queries of one portion, all heads; wave w has queries 4w .. 4w + 3. Heads sit in
// slots of 4 that share a key head (slot s: key head s / QPG, its heads 4 (s % QPG) ..,
// those past the group's end empty), so a row tile is the wave's 4 queries x a slot's heads.
//
// Per page: S = Q K^T slot by slot (K fragments are read some steps ahead of their
// MFMAs), the next K and this V on their way by LDS-DMA, mix and softmax, P through this
// wave's corner of LDS into operand order, P V. The outputs live in named AGPRs
// (acc_regs.h, accumulator s ND + d): they take half the register file, and the compiler
// would move them about. Rescales are collected over the page and applied before P V.
//
// Q is too large for what is left of the registers. Up to four slots, eight waves (two per
// SIMD) share K and V, and LDS has room for the first LQ row tiles' Q. Above, four waves
// have all registers, and RES row tiles' stay there. The others come from memory again
// for every page, the first of them during the last page's P V: what counts is that all
// workgroups of an XCD together fit its L2.
template <int NS>
constexpr int waves() { return NS <= 4 ? 8 : 4; }

template <int NS, int NK, int ND>
__global__ __launch_bounds__(64 * waves<NS>()) __attribute__((amdgpu_waves_per_eu(waves<NS>() / 4, waves<NS>() / 4)))
void attn_tiles(Args a) {
  constexpr int MT = (NS + 3) / 4, NW = waves<NS>();
  constexpr bool TWO = NW == 8;  // two waves per SIMD: half the registers
  constexpr int LQ = !TWO ? 0 : NS < 8 / NK ? NS : 8 / NK;
  constexpr int RQ = TWO ? 1 : NS * NK <= 16 ? NS : 16 / NK;  // row tiles' Q in registers
  constexpr int RES = TWO || NK == 2 ? 0 : 1, RB = RQ - RES;
  // register place of a row tile past LQ: the first RES for good, the others through a ring of RB
  auto ring = [](int rt) { return rt - LQ < RES ? rt - LQ : RES + (rt - LQ - RES) % RB; };
  static_assert(NS * ND <= 64, "outputs exceed the AGPRs");
  __shared__ __attribute__((aligned(1024))) char smem[(NS * (2 * NK + ND) + NW * (NS + LQ * NK)) * 1024];
  char* const ks = smem;
  char* const vs = smem + NS * 2 * NK * 1024;
  const int lane = threadIdx.x & 63, w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), n = lane & 15, q = lane >> 4;
  // where this lane reads V: an address of its own, within the reach of the reads' offsets
  unsigned vl = (unsigned)(uintptr_t)(KGS_LDS char*)vs + 16 * lane;
  asm volatile("" : "+v"(vl));
  char* const ps = vs + NS * ND * 1024 + w * NS * 1024;  // this wave's P: [slot][16 rows][32 keys]
  char* const lq = vs + NS * (ND + NW) * 1024 + w * LQ * NK * 1024 + 16 * lane;  // and its Q
  const int4 it = a.items[2 * blockIdx.x], part = a.items[2 * blockIdx.x + 1];  // part: first page, end, result (-1: whole)
  const int qpg = (a.R + 3) / 4, nslot = a.G * qpg;
  const int* bt = a.bt + (long)it.y * a.W;
  const int pend = part.y;
  constexpr int DK = 32 * NK, DV = 16 * ND, HPAGE = PAGE * (DK + DV) * 2;  // bytes of one head's page
  const int posw = it.z + 4 * w;                        // position of the wave's first query

  // this lane's row of the S tiles: query n >> 2 of the block, head n & 3 of the slot. A query
  // past the portion's end reads its last one; an empty head reads what follows the
  // group (zeros past the last row): its scale is 0.
  const __amdgpu_buffer_rsrc_t qrsrc = __builtin_amdgcn_make_buffer_rsrc((void*)((const unsigned short*)a.q + (long)it.x * a.ldq), 0,
                                                       it.w * (int)a.ldq * 2, 0x00020000);
  const int qoff = (min(4 * w + (n >> 2), it.w - 1) * (int)a.ldq + (n & 3) * DK + 8 * q) * 2;
  auto first_q = [&](bf16x8 (&f)[NK], int s) {
    const int so = (min(s / qpg, a.G - 1) * a.R + 4 * (s % qpg)) * DK * 2;
#pragma unroll
    for (int k = 0; k < NK; ++k)
      f[k] = __builtin_bit_cast(bf16x8, __builtin_amdgcn_raw_buffer_load_b128(qrsrc, qoff + 64 * k, so, 0));
  };
  // Those rows lie 16 to a load. They are read again for every page, so the wave puts them down
  // in operand order first, 1 KB a fragment.
  char* const qs = (char*)a.qs + ((long)blockIdx.x * NW + w) * (NS * NK * 1024);
  auto load_q = [&](bf16x8 (&f)[NK], int rt) {
#pragma unroll
    for (int k = 0; k < NK; ++k) f[k] = load_frag(qs, NS * NK * 1024, 16 * lane, (rt * NK + k) * 1024);
  };
  float sc[NS][4];  // uniform
#pragma unroll
  for (int s = 0; s < NS; ++s)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int hr = 4 * (s % qpg) + r;
      sc[s][r] = __uint_as_float(__builtin_amdgcn_readfirstlane(
          __float_as_uint(s < nslot && hr < a.R ? a.sc[s / qpg * a.R + hr] : 0.f)));
    }
  f16x8 tf[MT];
#pragma unroll
  for (int t = 0; t < MT; ++t) tf[t] = *(const f16x8*)(a.talk + (t * 64 + lane) * 8);

  // Every slot has a place for its key head's K and V. They come in chunks of 1 KB, dealt to the
  // waves: chunk w + NW c of `per` a slot.
  const int pbytes = a.G * HPAGE;
  int head[NS];  // where a slot's head begins in a page
#pragma unroll
  for (int s = 0; s < NS; ++s) head[s] = min(s / qpg, a.G - 1) * HPAGE;
  auto dma = [&](int page, char* dst, int per, int first, int c) {  // per: 4 or 8
    const int lo = NW * c / per, so = per < NW && w >= per ? head[lo + 1] : head[lo];
    dma_chunk((const char*)a.pages + (long)page * pbytes, pbytes, dst + (w + NW * c) * 1024, 16 * lane,
              so + first + (NW * c + w) % per * 1024);
  };
  constexpr int CK = NS * 2 * NK / NW, CV = NS * ND / NW;  // chunks per wave of K and of V
  constexpr int CV1 = CV / 2, CK1 = CK / 2;                // V: before the mixture and in it; K: in it and after
  constexpr int KPER = 2 * NK, VPER = ND;
  auto page_id = [&](int pg) { return bt[min(pg, pend - 1)]; };

  // the far bias less the running maximum of (query, slot 4t + q, head): the mixture's addend
  f32x4 cm[4][MT];
  float l[NS];
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int t = 0; t < MT; ++t) cm[i][t] = *(const f32x4*)(a.bfar + 16 * t + 4 * q);
#pragma unroll
  for (int i = 0; i < NS; ++i) l[i] = 0.f;
  if constexpr (TWO) KGS_ACC_RESERVE_HALF();
  else KGS_ACC_RESERVE();
  static_for<0, NS * ND>([](auto i) { accr::zero<decltype(i)::value>(); });

  bf16x8 qf[RQ][NK];
#pragma unroll
  for (int i = 0; i < LQ; ++i) {
    first_q(qf[0], i);
#pragma unroll
    for (int k = 0; k < NK; ++k) *(bf16x8*)(lq + (i * NK + k) * 1024) = qf[0][k];
  }
#pragma unroll
  for (int i = NS - 1; i >= LQ; --i) {
    first_q(qf[ring(i)], i);
#pragma unroll
    for (int k = 0; k < NK; ++k) *(bf16x8*)(qs + (i * NK + k) * 1024 + 16 * lane) = qf[ring(i)][k];
  }
  int page = __builtin_amdgcn_readfirstlane(page_id(part.x));
#pragma unroll
  for (int c = 0; c < CK; ++c) dma(page, ks, KPER, 0, c);
  bar<0>();
  for (int pg = part.x; pg < pend; ++pg) {
    const int tok0 = pg * PAGE;
    const int next = page_id(pg + 1);
    // ---- scores
    // A slot's scores become its fp16 parts while the next slot's MFMAs run.
    unsigned x[2][2][MT][2][4];  // [key half][part][half of the slots][head pair][slot of it, then query]
    f32x4 S[2][2];
    auto split_slot = [&](int s, int u0, int u1) {  // units u0 .. u1 - 1 of 4: (key half, head pair)
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        if (u < u0 || u >= u1) continue;
        const int kt = u >> 1, c = u & 1;
        const f32x4& v = S[s & 1][kt];
        unsigned &hi = x[kt][0][s >> 2][c][s & 3], &lo = x[kt][1][s >> 2][c][s & 3];
        split2(v[2 * c] * sc[s][2 * c], v[2 * c + 1] * sc[s][2 * c + 1], hi, lo);
        asm volatile("" : "+v"(hi), "+v"(lo));  // here, not where they are used
      }
    };
    if constexpr (NS < 4) {
#pragma unroll
      for (int i = 0; i < 8; ++i)
#pragma unroll
        for (int s = NS; s < 4; ++s) x[i >> 2][i >> 1 & 1][0][i & 1][s] = 0;
    }
    // K fragments of both 16-key halves, one 32-dim step at a time, PF steps ahead
    constexpr int PF = TWO ? 1 : 3, STEPS = NS * NK;
    bf16x8 kf[PF + 1][2], ql[PF + 1];
    auto read_k = [&](int p) {
      const char* kp = ks + (p / NK * 2 * NK + p % NK) * 1024 + 16 * lane;
      kf[p % (PF + 1)][0] = *(const bf16x8*)kp;
      kf[p % (PF + 1)][1] = *(const bf16x8*)(kp + NK * 1024);
      if (p / NK < LQ) ql[p % (PF + 1)] = *(const bf16x8*)(lq + p * 1024);
    };
#pragma unroll
    for (int p = 0; p < PF; ++p) read_k(p);
#pragma unroll
    for (int p = 0; p < STEPS; ++p) {
      if (p + PF < STEPS) read_k(p + PF);
      fence();
      const int s = p / NK;
      f32x4(&c)[2] = S[s & 1];
      if (p % NK == 0) c[0] = c[1] = f32x4{};
#pragma unroll
      for (int kt = 0; kt < 2; ++kt)
        c[kt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(s < LQ ? ql[p % (PF + 1)] : qf[s < LQ ? 0 : ring(s)][p % NK],
                                                        kf[p % (PF + 1)][kt], c[kt], 0, 0, 0);
      if (s > 0) split_slot(s - 1, p % NK * 4 / NK, (p % NK + 1) * 4 / NK);
      if (p % NK == NK - 1) {
        fence();
        if (s >= LQ + RES && s + RB < NS) load_q(qf[ring(s)], s + RB);
      }
#pragma unroll
      for (int c = 0; c < CV1; ++c)  // half of this page's V
        if (c * STEPS / (CV1 ? CV1 : 1) == p) dma(page, vs, VPER, PAGE * DK * 2, c);
      fence();
    }
    split_slot(NS - 1, 0, 4);
    bar<63>();  // K of this page is done with everywhere
    const int pnext = __builtin_amdgcn_readfirstlane(next);

    // ---- mix, softmax
    const bool near = posw - (tok0 + PAGE - 1) < a.nfar, edge = tok0 + PAGE - 1 > posw;
    bool grown = false;
    float al[NS];
#pragma unroll
    for (int i = 0; i < NS; ++i) al[i] = 1.f;
    {
      unsigned p0[4][MT][2];  // keys 2n, heads (0, 1) and (2, 3)
#pragma unroll
      for (int kt = 0; kt < 2; ++kt) {
#pragma unroll
        for (int j = 0; j < 2; ++j)
#pragma unroll
          for (int hf = 0; hf < MT; ++hf) transpose4(x[kt][j][hf][0]), transpose4(x[kt][j][hf][1]);
        f32x4 D[4][MT];
#pragma unroll
        for (int j = 1; j >= 0; --j)
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            const unsigned(&y)[MT][2][4] = x[kt][j];
            const u32x4 b = {y[0][0][i], y[0][1][i], MT > 1 ? y[MT - 1][0][i] : 0u, MT > 1 ? y[MT - 1][1][i] : 0u};
#pragma unroll
            for (int t = 0; t < MT; ++t)
              D[i][t] = __builtin_amdgcn_mfma_f32_16x16x32_f16(tf[t], __builtin_bit_cast(f16x8, b),
                                                               j == 1 ? cm[i][t] : D[i][t], 0, 0, 0);
          }
        // lane: query i, key 2n + kt, slot 4t + q, head r; above the running maximum
        const int dist = posw - (tok0 + 2 * n + kt);  // of query 0
        if (near) {
          // all loads, then all sums: waited for here, not where far pages pass too
          f32x4 b[4][MT];
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            const unsigned at = min(max(dist + i, 0), a.nfar) * a.ldb + 4 * q;
#pragma unroll
            for (int t = 0; t < MT; ++t) b[i][t] = *(const f32x4*)(a.bias + (at + 16 * t));
          }
          fence();
#pragma unroll
          for (int i = 0; i < 4; ++i)
#pragma unroll
            for (int t = 0; t < MT; ++t) {
              D[i][t] += b[i][t];
              asm volatile("" : "+v"(D[i][t]));
            }
        }
        if (edge) {
#pragma unroll
          for (int i = 0; i < 4; ++i)
#pragma unroll
            for (int t = 0; t < MT; ++t)
#pragma unroll
              for (int r = 0; r < 4; ++r) D[i][t][r] = dist + i < 0 ? NEG : D[i][t][r];
        }
        float over = D[0][0][0];
#pragma unroll
        for (int i = 0; i < 4; ++i)
#pragma unroll
          for (int t = 0; t < MT; ++t) over = fmaxf(fmaxf(fmaxf(over, D[i][t][0]), fmaxf(D[i][t][1], D[i][t][2])), D[i][t][3]);
        if (__builtin_expect(__any(over > RESCALE), 0)) {
          // new maxima over the 16 keys; sel: the factor of head n & 3, for the lanes that hold its row
          grown = true;
          int n_ = n;
          asm volatile("" : "+v"(n_));  // nothing of this path is worth a register outside it
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            float sel[MT];
#pragma unroll
            for (int t = 0; t < MT; ++t) {
              float fr[4];
#pragma unroll
              for (int r = 0; r < 4; ++r) {
                float up = fmaxf(D[i][t][r], 0.f);
#pragma unroll
                for (int b = 1; b < 16; b <<= 1)
                  up = fmaxf(up, __int_as_float(__builtin_amdgcn_ds_bpermute(((n_ ^ b) + 16 * q) * 4, __float_as_int(up))));
                fr[r] = __builtin_amdgcn_exp2f(-up);
                cm[i][t][r] -= up;
                D[i][t][r] -= up;
              }
              sel[t] = (n_ & 2) ? ((n_ & 1) ? fr[3] : fr[2]) : ((n_ & 1) ? fr[1] : fr[0]);
              if (kt == 1) {
#pragma unroll
                for (int c = 0; c < 2; ++c)
                  p0[i][t][c] = pack_bf16x2(__uint_as_float(p0[i][t][c] << 16) * fr[2 * c],
                                            __uint_as_float(p0[i][t][c] & 0xffff0000u) * fr[2 * c + 1]);
              }
            }
#pragma unroll
            for (int s = 0; s < NS; ++s) {
              const float g = __shfl(sel[s >> 2], 16 * (s & 3) + (n_ & 3), 64);
              al[s] *= (n_ >> 2) == i ? g : 1.f;
            }
          }
        }
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          // a chunk or two at a time: the rest of this page's V, then half of the next one's K
          fence();
#pragma unroll
          for (int c = CV1; c < CV + CK1; ++c)
            if ((c - CV1) * 8 / (CV - CV1 + CK1) == 4 * kt + i) {
              if (c < CV) dma(page, vs, VPER, PAGE * DK * 2, c);
              else dma(pnext, ks, KPER, 0, c - CV);
            }
#pragma unroll
          for (int t = 0; t < MT; ++t) {
            float p[4];
#pragma unroll
            for (int r = 0; r < 4; ++r) p[r] = __builtin_amdgcn_exp2f(D[i][t][r]);
            const unsigned c0 = pack_bf16x2(p[0], p[1]), c1 = pack_bf16x2(p[2], p[3]);
            if (kt == 0) p0[i][t][0] = c0, p0[i][t][1] = c1;
            else if (NS >= 4 || q < NS) {
              // row 4i + r of slot 4t + q, keys 2n and 2n + 1; rows permuted by the slot and 16-B
              // chunks by the row: no bank twice
              char* pp = ps + (4 * t + q) * 1024 + 256 * i + (((n >> 2) ^ i) * 16) + (n & 3) * 4;
              *(unsigned*)(pp + ((0 ^ q) * 64)) = __builtin_amdgcn_perm(c0, p0[i][t][0], 0x05040100u);
              *(unsigned*)(pp + ((1 ^ q) * 64)) = __builtin_amdgcn_perm(c0, p0[i][t][0], 0x07060302u);
              *(unsigned*)(pp + ((2 ^ q) * 64)) = __builtin_amdgcn_perm(c1, p0[i][t][1], 0x05040100u);
              *(unsigned*)(pp + ((3 ^ q) * 64)) = __builtin_amdgcn_perm(c1, p0[i][t][1], 0x07060302u);
            }
          }
        }
      }
    }
    if (__builtin_expect(grown, 0)) {
      asm volatile("s_nop 7\n\ts_nop 7\n\ts_nop 3" ::: "memory");  // MFMA -> v_accvgpr_read hazard
      static_for<0, NS>([&](auto rc) {
        constexpr int s = decltype(rc)::value;
        l[s] *= al[s];
        static_for<0, ND>([&](auto dc) {
          constexpr int i = s * ND + decltype(dc)::value;
          accr::write<i>(accr::read<i>() * al[s]);
        });
      });
      asm volatile("s_nop 7" ::: "memory");
    }
    bar<CK1>();  // V of this page is there
    page = pnext;

    // ---- P V
#pragma unroll
    for (int i = RES; i < RQ; ++i)
      if (LQ + i < NS) load_q(qf[i], LQ + i);  // for the next page
    constexpr int VB = TWO ? 1 : 2;  // slots' V in registers
    bf16x8 vf[VB][ND];
    auto read_v = [&](bf16x8 (&f)[ND], int s) {
#pragma unroll
      for (int i = 0; i < ND; ++i) f[i] = *(const KGS_LDS bf16x8*)(uintptr_t)(vl + (s * ND + i) * 1024);
    };
    u32x4 pw[VB];
    auto read_p = [&](u32x4& f, int s) {
      f = *(const u32x4*)(ps + s * 1024 + ((n ^ (s & 3)) * 64) + ((q ^ ((n >> 2) & 3)) * 16));
    };
    read_p(pw[0], 0);
    read_v(vf[0], 0);
    fence();
    static_for<0, NS>([&](auto sc_) {
      constexpr int s = decltype(sc_)::value;
      if constexpr (TWO && s > 0) {
        read_p(pw[0], s);
        read_v(vf[0], s);
      } else if constexpr (!TWO && s + 1 < NS) {
        read_p(pw[(s + 1) & 1], s + 1);
        read_v(vf[(s + 1) & 1], s + 1);
      }
      fence();
#pragma unroll
      for (int c = CK1; c < CK; ++c)  // the other half of K (past the last page: that one again)
        if ((c - CK1) * NS / 2 / (CK - CK1) == s) dma(pnext, ks, KPER, 0, c);
      const u32x4 pv = pw[s % VB];
      const bf16x8 pb = __builtin_bit_cast(bf16x8, pv);
      static_for<0, ND>([&](auto dc) {
        constexpr int d = decltype(dc)::value;
        accr::mfma<s * ND + d>(vf[s % VB][d], pb);
      });
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const unsigned two = pv[e], ones = 0x3f803f80u;
        l[s] = __builtin_amdgcn_fdot2_f32_bf16(__builtin_bit_cast(bf16x2, two), __builtin_bit_cast(bf16x2, ones), l[s], false);
      }
      fence();
    });
    bar<0>();  // V is done with everywhere, K of the next page is there
  }

  // rows' maxima to the lanes that hold the rows: [slot][row]
  float* mm = (float*)ps;
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int t = 0; t < MT; ++t)
      if (NS >= 4 || q < NS) *(f32x4*)(mm + (4 * t + q) * 16 + 4 * i) =
                                  *(const f32x4*)(a.bfar + 16 * t + 4 * q) - cm[i][t];
  asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
  asm volatile("s_nop 7\n\ts_nop 7\n\ts_nop 3" ::: "memory");  // MFMA -> v_accvgpr_read hazard
  static_for<0, NS>([&](auto sc_) {
      constexpr int s = decltype(sc_)::value;
      const int hr = 4 * (s % qpg) + (n & 3), qi = 4 * w + (n >> 2);
      const float m = mm[s * 16 + n], L = xor32_sum(xor16_sum(l[s]));
      const bool ok = s < nslot && hr < a.R && qi < it.w;
      const int h = s / qpg * a.R + hr;
      if (part.z < 0) {
        const float inv = 1.0f / (L + __builtin_amdgcn_exp2f(-m));
        unsigned short* op = (unsigned short*)a.o + (long)(it.x + qi) * a.ldo + (long)h * DV + 4 * q;
        static_for<0, ND>([&](auto dc) {
          constexpr int d = decltype(dc)::value;
          const f32x4 o = accr::read<s * ND + d>() * inv;
          uint2 pk;
          pk.x = pack_bf16x2(o[0], o[1]);
          pk.y = pack_bf16x2(o[2], o[3]);
          if (ok) *(uint2*)(op + 16 * d) = pk;
        });
      } else {
        const long pr = ((long)part.z * (4 * NW) + qi) * a.H + h;
        static_for<0, ND>([&](auto dc) {
          constexpr int d = decltype(dc)::value;
          const f32x4 o = accr::read<s * ND + d>();
          if (ok) *(f32x4*)(a.po + pr * DV + 16 * d + 4 * q) = o;
        });
        if (ok && q == 0) a.pml[2 * pr] = m, a.pml[2 * pr + 1] = L;
      }
  });
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
  if (a.nsplit > 1) hipLaunchKernelGGL(merge<false>, dim3((unsigned)(nrows * a.H)), dim3(64), 0, s, a);
}
template <int NK, int ND>
void rows_ht(const Args& a, int nrows, hipStream_t s) {
  if (a.H <= 16) run_rows<1, NK, ND>(a, nrows, s);
  else if (a.H <= 32) run_rows<2, NK, ND>(a, nrows, s);
  else run_rows<4, NK, ND>(a, nrows, s);
}
template <int NK, int ND>
void tiles_ns(const Args& a, int nitems, int nslot, hipStream_t s) {
  const dim3 grid((unsigned)nitems);
  if (nslot <= 2) hipLaunchKernelGGL((attn_tiles<2, NK, ND>), grid, dim3(64 * waves<2>()), 0, s, a);
  else if (nslot <= 4) hipLaunchKernelGGL((attn_tiles<4, NK, ND>), grid, dim3(64 * waves<4>()), 0, s, a);
  else hipLaunchKernelGGL((attn_tiles<8, NK, ND>), grid, dim3(64 * waves<8>()), 0, s, a);
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
// b their biases one after another (nq + G dkp + G dvp), or null. q += b in place, k + b and
// v + b go to their slots. wq, wk not null: q and k normed per seg columns (dkp or a part of it;
// dim without padding). cs not null: q and k rotated by the row's position, the
// pairs (0, 1), (2, 3), .. of each seg's first `rot` dims by cs [npos][rot / 2][cos, sin].
// every > 0: q times 1 + coef ln(floor((pos + 1) / every) + 1).
KGS_EXPORT int kgs_talking_write(void* z, long ldz, const void* b, void* pages, const void* slots, int T, int nq, int G,
                                 int dkp, int dvp, int ok, int ov, const void* cs, const void* pos, int npos, int rot,
                                 const void* wq, const void* wk, int seg, int dim, float eps, float coef, int every,
                                 int f32, hipStream_t s) {
  using namespace kgs::talking;
  if (T <= 0 || nq <= 0 || G <= 0 || dkp <= 0 || dvp <= 0 || dkp % 32 || dvp % 16 || nq % 8 || ok < nq ||
      ldz < ok + G * dkp || ldz < ov + G * dvp || T > 8 * 65535)
    return KGS_ERR_SHAPE;
  if (seg <= 0 || seg % 8 || dkp % seg || dim <= 0 || dim > seg || every < 0 || (every && !pos) || !wq != !wk)
    return KGS_ERR_SHAPE;
  if (wq && (seg > 2048 || nq % dkp)) return KGS_ERR_SHAPE;
  if (ldz % 8 || ok % 8 || ov % 8 || (((uintptr_t)z | (uintptr_t)pages | (uintptr_t)b) & 15)) return KGS_ERR_ALIGN;
  if (cs && (!pos || npos <= 0 || rot <= 0 || rot % 8 || rot > seg || nq % dkp)) return KGS_ERR_SHAPE;
  if ((uintptr_t)cs & 15) return KGS_ERR_ALIGN;
  WriteArgs a{z, ldz, (const float*)b, pages, (const int*)slots, T, nq, G, dkp, dvp, ok, ov,
              (const float*)cs, (const int*)pos, npos, rot, (const float*)wq, (const float*)wk, seg, dim, eps, coef, every};
  const int n = (nq + G * (dkp + dvp)) / 8;
  const int norm = !wq ? 0 : seg == 64 ? 8 : seg == 128 ? 16 : 1, wg = norm == 1 ? 256 / (seg / 8) * (seg / 8) : 256;
  const dim3 grid((n + wg - 1) / wg, (T + 7) / 8);
  auto fn = f32 ? (norm == 0 ? write_kv<float, 0> : norm == 8 ? write_kv<float, 8> : norm == 16 ? write_kv<float, 16> : write_kv<float, 1>)
                : (norm == 0 ? write_kv<unsigned short, 0> : norm == 8 ? write_kv<unsigned short, 8>
                   : norm == 16 ? write_kv<unsigned short, 16> : write_kv<unsigned short, 1>);
  hipLaunchKernelGGL(fn, grid, dim3(256), 0, s, a);
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
         nullptr, 0, nullptr, (float*)po, (float*)pml, (const float*)sc, (const unsigned short*)talk, (const float*)talk, (const float*)bias,
         nullptr, ldb, nfar, H, G, G ? H / G : 0, dkp, dvp, nsplit};
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

// Prompt portions: nitems blocks of consecutive queries over a range of their pages, two
// int4 each (Args::items): up to 32 queries, 16 above 4 slots. A block split over its pages
// leaves partial results (po, pml: one part holds 32 or 16 rows of all heads) that
// `merges` names. bf16, dkp and dvp 64 or 128, at most 8 slots of 4 heads
// (G ceil(H / G / 4)); talk (fp16) and biases in slot order, ldb = 16 ceil(slots / 4); bias is
// the table less its last row, bfar. qs: scratch, slots (2, 4 or 8) x 4 KB x dkp / 32 per
// item, twice that up to 4 slots.
KGS_EXPORT int kgs_talking_tiles(const void* q, long ldq, const void* pages, void* o, long ldo, const void* bt, int W,
                                 const void* items, int nitems, const void* merges,
                                 int nmerge, void* po, void* pml, void* qs, const void* sc, const void* talk, const void* bias,
                                 const void* bfar, int ldb, int nfar, int H, int G, int dkp, int dvp, hipStream_t s) {
  using namespace kgs::talking;
  Args a{};
  a.q = q, a.ldq = ldq, a.pages = pages, a.o = o, a.ldo = ldo, a.bt = (const int*)bt, a.W = W;
  a.items = (const int4*)items, a.merges = (const int4*)merges, a.po = (float*)po, a.pml = (float*)pml, a.qs = qs, a.sc = (const float*)sc, a.talk = (const unsigned short*)talk;
  a.bias = (const float*)bias, a.bfar = (const float*)bfar, a.ldb = ldb, a.nfar = nfar, a.H = H, a.G = G, a.R = G ? H / G : 0;
  a.dkp = dkp, a.dvp = dvp, a.nsplit = 1;
  if (int rc = check(a, nitems)) return rc;
  const int nslot = G * ((H / G + 3) / 4);
  if (nslot > 8 || (dkp != 64 && dkp != 128) || (dvp != 64 && dvp != 128)) return KGS_ERR_ARG;
  if (ldb < (nslot + 3) / 4 * 16 || (((uintptr_t)items | (uintptr_t)bfar | (uintptr_t)talk | (uintptr_t)qs) & 15)) return KGS_ERR_SHAPE;
  a.tile = nslot <= 4 ? 32 : 16;
  if (nmerge < 0 || (nmerge && (!merges || !po || !pml)) || (long)nmerge * a.tile * H > 0x7fffffff) return KGS_ERR_SHAPE;
  if (dkp == 64) dvp == 64 ? tiles_ns<2, 4>(a, nitems, nslot, s) : tiles_ns<2, 8>(a, nitems, nslot, s);
  else dvp == 64 ? tiles_ns<4, 4>(a, nitems, nslot, s) : tiles_ns<4, 8>(a, nitems, nslot, s);
  if (nmerge) hipLaunchKernelGGL(merge<true>, dim3((unsigned)(nmerge * a.tile / 4 * H)), dim3(256), 0, s, a);  // tile: whole 4s
  return (int)hipGetLastError();
}
