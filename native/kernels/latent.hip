// Latent attention: a token's keys and values of every head are linear maps of
// one small vector c (the latent), and only c is cached, in pages
// [page][32 tokens][RP] (RP: the latent size padded to a kernel size, pad zero). Where
// keys also have a part that turns with the position, one for all heads, its HR columns
// (padded, neighbouring pairs) follow the latent's, turned: a row is [c | kr].
//
// The absorbed form needs no expanded keys or values: with
//   qlat_h = W_uk,h^T q_h        score_j = (qlat_h . c_j + qr_h . kr_j) * scale
//   olat_h = sum_j p_j c_j       o_h     = W_uv,h olat_h
// attention is multi-query over c itself, every head (and every query token of a
// prompt portion) a row over the same keys. With a window of `win` positions a query sees
// itself and the win - 1 keys before it, and reads only their pages. Kernels:
//   * latent_norm   the RMS norms of both latents of a token's fused input
//                   projection; c goes straight into its cache slot, kr turned beside it;
//   * head_proj     the per-head products (W_uk^T q with qr turned beside it, W_uv olat),
//                   the latter with the sigmoid output gate (a number per head or per
//                   element) in its store;
//   * attn          rows x pages on v_mfma_f32_16x16x32_bf16, split over the
//                   context, + merge;
//   * attn_simple   the same on the VALU for any RP and for fp32 caches.
#include <type_traits>

#include "kgs_common.h"

namespace kgs {
namespace latent {

constexpr int PAGE = 32;
constexpr float NEG = -1.0e30f;
constexpr float RESCALE = 8.0f;  // deferred-max threshold, log2 units

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

__device__ __forceinline__ float wave_max(float v) {
#pragma unroll
  for (int m = 8; m >= 1; m >>= 1) v = fmaxf(v, __shfl_xor(v, m, 64));
  return xor32_max(xor16_max(v));
}
__device__ __forceinline__ float sigmoid(float x) { return 1.0f / (1.0f + expf(-x)); }

// ---------------------------------------------------------------- latent_norm
struct NormArgs {
  const void* z;  // [T, ldz] fused input projection
  long ldz;
  int oq, nq, qp;  // query latent: first column, size, padded size of cq
  int oc, nc, rp;  // key/value latent (nc 0: the layer has none of its own)
  int okr, hr;     // rotated key part: first column, padded size (0: none)
  const float* cs; // [npos][rot]: cos and sin of each pair
  const int* pos;  // [T]
  int npos, rot;
  const float *wq, *wc;
  void* cq;              // [T, qp]
  void* cache;           // this layer's pages
  const int* slots;      // [T], -1: not cached
  float eps;
};

__device__ __forceinline__ const float* turns(const float* cs, int pos, int npos, int rot) {
  return cs + (long)min(max(pos, 0), npos - 1) * rot;
}

// workgroup (token, 0): the query latent, (token, 1): the cached one; up to
// NORM_REG values per thread stay in registers between the sum and the scaling
constexpr int NORM_REG = 8;

// bf16 rows in 16-B pieces: one wave per (token, latent), NV pieces per lane
constexpr int NORM_NV = 4;  // up to 2048 values
__global__ __launch_bounds__(256) void norm_vec(NormArgs a, int T) {
  const int lane = threadIdx.x & 63;
  const long t = (long)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (t >= T) return;
  const bool second = blockIdx.y == 1;
  const int n = second ? a.nc : a.nq, np = second ? a.rp : a.qp;
  const int slot = second ? a.slots[t] : 0;
  if (slot < 0) return;
  const unsigned short* z = (const unsigned short*)a.z + t * a.ldz + (second ? a.oc : a.oq);
  const float* w = second ? a.wc : a.wq;
  unsigned short* out =
      second ? (unsigned short*)a.cache + (long)slot * (a.rp + a.hr) : (unsigned short*)a.cq + t * a.qp;
  if (second && 8 * lane < a.hr) {
    const bf16x8 u = *(const bf16x8*)((const unsigned short*)a.z + t * a.ldz + a.okr + 8 * lane);
    float y[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) y[j] = bf2f((unsigned short)u[j]);
    if (8 * lane < a.rot) {
      const float* p = turns(a.cs, a.pos[t], a.npos, a.rot) + 8 * lane;
#pragma unroll
      for (int j = 0; j < 8; j += 2) {
        const float v = y[j], w2 = y[j + 1];
        y[j] = rope_lo(v, w2, p[j], p[j + 1]);
        y[j + 1] = rope_hi(v, w2, p[j], p[j + 1]);
      }
    }
    *(bf16x8*)(out + a.rp + 8 * lane) = pack_bf16x8(y, 0);
  }
  bf16x8 x[NORM_NV];
  f32x4 wv[NORM_NV][2];  // loaded ahead of the sum
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < NORM_NV; ++i) {
    const int c = 8 * (lane + 64 * i);
    if (c < n) {
      x[i] = *(const bf16x8*)(z + c);
      wv[i][0] = *(const f32x4*)(w + c);
      wv[i][1] = *(const f32x4*)(w + c + 4);
    } else {
      x[i] = bf16x8{};
      wv[i][0] = f32x4{};
      wv[i][1] = f32x4{};
    }
  }
#pragma unroll
  for (int i = 0; i < NORM_NV; ++i)
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const float v = bf2f((unsigned short)x[i][j]);
      ss = __builtin_fmaf(v, v, ss);
    }
  const float r = 1.0f / sqrtf(wave_sum(ss) / n + a.eps);
#pragma unroll
  for (int i = 0; i < NORM_NV; ++i) {
    const int c = 8 * (lane + 64 * i);
    if (c >= np) continue;
    float y[8];
#pragma unroll
    for (int j = 0; j < 8; ++j) y[j] = bf2f((unsigned short)x[i][j]) * r * wv[i][j >> 2][j & 3];
    *(bf16x8*)(out + c) = pack_bf16x8(y, 0);
  }
}

template <typename T>
__global__ __launch_bounds__(256) void norm(NormArgs a) {
  __shared__ float red[4];
  const int tid = threadIdx.x;
  const long t = blockIdx.x;
  const bool second = blockIdx.y == 1;
  const int n = second ? a.nc : a.nq, np = second ? a.rp : a.qp;
  const int slot = second ? a.slots[t] : 0;
  if (slot < 0) return;
  const T* z = (const T*)a.z + t * a.ldz + (second ? a.oc : a.oq);
  const float* w = second ? a.wc : a.wq;
  T* out = second ? (T*)a.cache + (long)slot * (a.rp + a.hr) : (T*)a.cq + t * a.qp;
  if (second) {
    const T* zr = (const T*)a.z + t * a.ldz + a.okr;
    for (int c = 2 * tid; c < a.hr; c += 512) {
      const float u = ld(zr + c), v = ld(zr + c + 1);
      float cs = 1.f, sn = 0.f;
      if (c < a.rot) {
        const float* p = turns(a.cs, a.pos[t], a.npos, a.rot) + c;
        cs = p[0], sn = p[1];
      }
      st(out + a.rp + c, rope_lo(u, v, cs, sn));
      st(out + a.rp + c + 1, rope_hi(u, v, cs, sn));
    }
  }
  float x[NORM_REG], ss = 0.f;
#pragma unroll
  for (int i = 0; i < NORM_REG; ++i) {
    const int c = tid + 256 * i;
    x[i] = c < n ? ld(z + c) : 0.f;
    ss += x[i] * x[i];
  }
  for (int c = tid + 256 * NORM_REG; c < n; c += 256) {
    const float v = ld(z + c);
    ss += v * v;
  }
  ss = wave_sum(ss);
  if ((tid & 63) == 0) red[tid >> 6] = ss;
  __syncthreads();
  const float r = 1.0f / sqrtf((red[0] + red[1] + red[2] + red[3]) / n + a.eps);
#pragma unroll
  for (int i = 0; i < NORM_REG; ++i) {
    const int c = tid + 256 * i;
    if (c < np) st(out + c, c < n ? x[i] * r * w[c] : 0.f);
  }
  for (int c = tid + 256 * NORM_REG; c < np; c += 256) st(out + c, c < n ? ld(z + c) * r * w[c] : 0.f);
}

// ------------------------------------------------------------------ head_proj
struct ProjArgs {
  const void* a;     // input row of token i, head h: a + in_row(i) * lda + h * ha
  const void* w;     // [H][N][K]
  void* out;         // out + out_row(i) * ldo + h * ho
  const int *idx_in, *idx_out;  // token i's row, or null (i)
  const void* gate;  // [rows, ldg] per output row: head h at column h hg, output n at n eg more; or null
  long lda, ha, ldo, ho, ldg;
  int hg, eg;
  int Nt, H, N, K;
  // hr columns after the K inputs, turned by the token's position, go after the N outputs
  int hr, npos, rot;
  const float* cs;
  const int* pos;  // [Nt]
};

// D^T[n][token] = W[n][k] a^T[k][token]; wave: 16 outputs x 16 TT tokens of one head
template <int TT>
__global__ __launch_bounds__(256) void head_proj(ProjArgs p) {
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
  const int l16 = lane & 15, g = lane >> 4;
  const int nt = blockIdx.x * 4 + w, h = blockIdx.z, t0 = blockIdx.y * 16 * TT;
  if (nt * 16 >= p.N) {
    const int c = nt * 16 - p.N + 4 * g;
    if (c >= p.hr) return;
#pragma unroll
    for (int i = 0; i < TT; ++i) {
      const int t = t0 + 16 * i + l16;
      if (t >= p.Nt) continue;
      const long ri = p.idx_in ? p.idx_in[t] : t, ro = p.idx_out ? p.idx_out[t] : t;
      const bf16x4 u = *(const bf16x4*)((const unsigned short*)p.a + ri * p.lda + h * p.ha + p.K + c);
      float y[4];
#pragma unroll
      for (int j = 0; j < 4; ++j) y[j] = bf2f((unsigned short)u[j]);
      if (c < p.rot) {
        const f32x4 cs = *(const f32x4*)(turns(p.cs, p.pos[t], p.npos, p.rot) + c);
#pragma unroll
        for (int j = 0; j < 4; j += 2) {
          const float v = y[j], x = y[j + 1];
          y[j] = rope_lo(v, x, cs[j], cs[j + 1]);
          y[j + 1] = rope_hi(v, x, cs[j], cs[j + 1]);
        }
      }
      uint2 o;
      o.x = pack_bf16x2(y[0], y[1]);
      o.y = pack_bf16x2(y[2], y[3]);
      *(uint2*)((unsigned short*)p.out + ro * p.ldo + h * p.ho + p.N + c) = o;
    }
    return;
  }
  const unsigned short* wp = (const unsigned short*)p.w + ((long)h * p.N + nt * 16 + l16) * p.K + 8 * g;
  const unsigned short* ap[TT];
#pragma unroll
  for (int i = 0; i < TT; ++i) {
    int t = t0 + 16 * i + l16;
    t = t < p.Nt ? t : p.Nt - 1;
    const long r = p.idx_in ? p.idx_in[t] : t;
    ap[i] = (const unsigned short*)p.a + r * p.lda + h * p.ha + 8 * g;
  }
  f32x4 acc[TT];
#pragma unroll
  for (int i = 0; i < TT; ++i) acc[i] = f32x4{};
  for (int k = 0; k < p.K; k += 128) {  // four steps' loads are in flight together
    bf16x8 wf[4], af[4][TT];
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (k + 32 * j < p.K) {
        wf[j] = *(const bf16x8*)(wp + k + 32 * j);
#pragma unroll
        for (int i = 0; i < TT; ++i) af[j][i] = *(const bf16x8*)(ap[i] + k + 32 * j);
      }
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (k + 32 * j < p.K) {
#pragma unroll
        for (int i = 0; i < TT; ++i)
          acc[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[j], af[j][i], acc[i], 0, 0, 0);
      }
  }
#pragma unroll
  for (int i = 0; i < TT; ++i) {
    const int t = t0 + 16 * i + l16;
    if (t >= p.Nt) continue;
    const long r = p.idx_out ? p.idx_out[t] : t;
    f32x4 s = f32x4{1.0f, 1.0f, 1.0f, 1.0f};
    if (p.gate) {
      const unsigned short* gp = (const unsigned short*)p.gate + r * p.ldg + (long)h * p.hg + (nt * 16 + 4 * g) * p.eg;
#pragma unroll
      for (int j = 0; j < 4; ++j) s[j] = sigmoid(bf2f(gp[j * p.eg]));
    }
    uint2 o;
    o.x = pack_bf16x2(acc[i][0] * s[0], acc[i][1] * s[1]);
    o.y = pack_bf16x2(acc[i][2] * s[2], acc[i][3] * s[3]);
    *(uint2*)((unsigned short*)p.out + r * p.ldo + h * p.ho + nt * 16 + 4 * g) = o;
  }
}

__global__ __launch_bounds__(256) void head_proj_f32(ProjArgs p) {
  const int i = blockIdx.x, h = blockIdx.y;
  const long ri = p.idx_in ? p.idx_in[i] : i, ro = p.idx_out ? p.idx_out[i] : i;
  const float* a = (const float*)p.a + ri * p.lda + h * p.ha;
  float* o = (float*)p.out + ro * p.ldo + h * p.ho;
  for (int c = 2 * threadIdx.x; c < p.hr; c += 512) {
    const float u = a[p.K + c], v = a[p.K + c + 1];
    float cs = 1.f, sn = 0.f;
    if (c < p.rot) {
      const float* t = turns(p.cs, p.pos[i], p.npos, p.rot) + c;
      cs = t[0], sn = t[1];
    }
    o[p.N + c] = rope_lo(u, v, cs, sn);
    o[p.N + c + 1] = rope_hi(u, v, cs, sn);
  }
  for (int n = threadIdx.x; n < p.N; n += 256) {
    const float s = p.gate ? sigmoid(((const float*)p.gate)[ro * p.ldg + (long)h * p.hg + n * p.eg]) : 1.0f;
    const float* w = (const float*)p.w + ((long)h * p.N + n) * p.K;
    float acc = 0.f;
    for (int k = 0; k < p.K; ++k) acc = __builtin_fmaf(a[k], w[k], acc);
    o[n] = acc * s;
  }
}

// ----------------------------------------------------------------------- attn
// Query tokens of the call are numbered 0 .. Nt - 1; sequence b holds tokens
// q0[b] .. q0[b] + n[b] - 1 at positions pos0[b] .. , its pages in bt[b].
struct Args {
  const void* q;      // [Nt * H, RP + HR]
  const void* cache;  // [pages][32][RP + HR]
  void* o;            // [Nt * H, RP]
  float* part_o;      // [nsplit][Nt * H][RP]
  float* part_ml;     // [nsplit][Nt * H][2]
  const int *q0, *n, *pos0, *bt;
  const int* items;   // (sequence, tile) pairs, or null: blockIdx.x = b * tiles + tile
  const int *tok_seq, *tok_pos;  // attn_simple
  int H, W, tiles, nsplit, Nt, RP, HR;
  float scale, sl2;  // sl2 = scale * log2(e)
  int win;           // 0: every earlier key
};

__device__ __forceinline__ int first_key(const Args& a, int pos) { return a.win ? max(0, pos - a.win + 1) : 0; }

template <int I, int N, class F>
__device__ __forceinline__ void static_for(F f) {
  if constexpr (I < N) {
    f(std::integral_constant<int, I>{});
    static_for<I + 1, N>(f);
  }
}

// a cache row: 32 RT latent columns (keys and values), 32 RK rotated ones (keys)
template <int RT, int RK>
struct Geo {
  static constexpr int RP = 32 * RT, KT = RT + RK, QP = 32 * KT, CH = 4 * KT, PITCH = 64 * KT, PAGEB = PAGE * PITCH;
  static constexpr int LOW = CH & -CH, P = LOW > 16 ? 16 : LOW;
  static constexpr int NP = P / 4;             // column steps whose swizzled addresses differ in more than an offset
  // pages in the ring: two workgroups per CU up to 384, one at 512
  static constexpr int NB = RT == 16 || 4 * PAGEB <= 80 * 1024 ? 4 : 3 * PAGEB <= 80 * 1024 ? 3 : 2;
  // XOR of a row's 16-B chunk index: rows that share banks land on other chunks
  __device__ static __forceinline__ int swz(int r) {
    if constexpr (P == 16) return ((r & 3) << 2) | ((r >> 1) & 2) | ((r >> 3) & 1);
    else if constexpr (P == 8) return (r >> 1) & 7;
    else return (r >> 2) & 3;
  }
  __device__ static __forceinline__ int off(int r, int c) { return PITCH * r + 16 * (c ^ swz(r)); }
};

// LDS reads by hand, several batches ahead of their MFMAs: a wave has its SIMD to
// itself here, so nothing else hides their latency, and the compiler takes a
// transposed read for a reader of the page being filled and would wait for the
// whole DMA in front of it. wait<N>: all but the N newest LDS operations are done.

// one 32-column step of a page's keys 0-15 and 16-31 (A operands)
struct KeyBatch {
  bf16x8 f[2];
  // at: address of step k % NP
  template <class G, int K>
  __device__ __forceinline__ void read(unsigned at) {
    constexpr int o = 16 * G::P * (K / G::NP);
    asm volatile("ds_read_b128 %0, %2 offset:%3\n\tds_read_b128 %1, %2 offset:%4"
                 : "=&v"(f[0]), "=&v"(f[1])
                 : "v"(at), "n"(o), "n"(o + 16 * G::PITCH));
  }
  template <int N>
  __device__ __forceinline__ void wait() {
    asm volatile("s_waitcnt lgkmcnt(%2)" : "+v"(f[0]), "+v"(f[1]) : "n"(N));
  }
};

// Two 16-column tiles of a page's 32 keys, transposed: four ds_read_b64_tr_b16
// (keys k0 .. and 16 + k0 .. of each), see tr_frag
struct TrBatch {
  bf16x4 lo[2], hi[2];
  // at: addresses of the two tiles of step j % NP
  template <class G, int J>
  __device__ __forceinline__ void read(const unsigned (&at)[2]) {
    constexpr int o = 16 * G::P * (J / G::NP);
#pragma unroll
    for (int x = 0; x < 2; ++x)
      asm volatile("ds_read_b64_tr_b16 %0, %2 offset:%3\n\tds_read_b64_tr_b16 %1, %2 offset:%4"
                   : "=&v"(lo[x]), "=&v"(hi[x])
                   : "v"(at[x]), "n"(o), "n"(o + 16 * G::PITCH));
  }
  template <int N>
  __device__ __forceinline__ void wait() {
    asm volatile("s_waitcnt lgkmcnt(%4)" : "+v"(lo[0]), "+v"(hi[0]), "+v"(lo[1]), "+v"(hi[1]) : "n"(N));
  }
  __device__ __forceinline__ bf16x8 frag(int x) const {
    return __builtin_shufflevector(lo[x], hi[x], 0, 1, 2, 3, 4, 5, 6, 7);
  }
};

// one wave's part of a page into its slot of the ring, swizzled
template <class G>
__device__ __forceinline__ void page_dma(const unsigned short* page, char* dst, int w, int nw, int lane) {
  const __amdgpu_buffer_rsrc_t src = __builtin_amdgcn_make_buffer_rsrc((void*)page, 0, G::PAGEB, 0x00020000);
#pragma unroll 4
  for (int i = w; i < 2 * G::KT; i += nw) {
    const int L = 64 * i + lane, r = L / G::CH, c = (L % G::CH) ^ G::swz(r);
    __builtin_amdgcn_raw_ptr_buffer_load_lds(src, (KGS_LDS void*)(dst + 1024 * i), 16, r * G::PITCH + 16 * c, 0, 0, 0);
  }
}

// All but the n newest vector memory operations of this wave are done (or fewer left).
__device__ __forceinline__ void vm_wait(int n) {
  if (n >= 32) asm volatile("s_waitcnt vmcnt(32)" ::: "memory");
  else if (n >= 24) asm volatile("s_waitcnt vmcnt(24)" ::: "memory");
  else if (n >= 16) asm volatile("s_waitcnt vmcnt(16)" ::: "memory");
  else if (n >= 12) asm volatile("s_waitcnt vmcnt(12)" ::: "memory");
  else if (n >= 8) asm volatile("s_waitcnt vmcnt(8)" ::: "memory");
  else if (n >= 4) asm volatile("s_waitcnt vmcnt(4)" ::: "memory");
  else if (n >= 2) asm volatile("s_waitcnt vmcnt(2)" ::: "memory");
  else asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
}

// Workgroup: 16 rows per wave of one sequence's (token, head) rows, head fastest,
// over the pages of one context split. S^T = C Q^T, so a lane owns row
// (lane & 15) and keys 16 t + 4 (lane >> 4) + r of a page; the same registers
// are the B operand of O^T = C^T P^T, whose A operand is the page read
// transposed (ds_read_b64_tr_b16) in that key order. Pages come through a ring of
// NB, NB - 1 of them in flight; one barrier per page says both that it has landed
// for every wave and that the page before it has been read by every wave.
template <int RT, int RK>
__global__ __launch_bounds__(RT > 8 ? 256 : 512) void attn(Args a) {
  using G = Geo<RT, RK>;
  extern __shared__ __attribute__((aligned(16))) char smem[];  // NB pages
  const int lane = threadIdx.x & 63, nw = blockDim.x >> 6;
  const int w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int l16 = lane & 15, g = lane >> 4, tq = (lane >> 2) & 3, tp = lane & 3;
  int b, tile;  // uniform: page ids then come by scalar loads
  if (a.items) {
    b = a.items[2 * blockIdx.x];
    tile = a.items[2 * blockIdx.x + 1];
  } else {
    b = __builtin_amdgcn_readfirstlane(blockIdx.x / a.tiles);
    tile = blockIdx.x - b * a.tiles;
  }
  const int rows = a.n[b] * a.H, pos0 = a.pos0[b];
  const long base = (long)a.q0[b] * a.H;  // row 0 of the sequence
  const int r0 = tile * 16 * nw;          // the workgroup's rows
  if (r0 >= rows) return;
  const int last = min(r0 + 16 * nw, rows) - 1;
  const int myrow = r0 + 16 * w + l16;
  const int row = min(myrow, last);
  const int pos = pos0 + row / a.H, lo = first_key(a, pos);
  const int wmax = pos0 + min(r0 + 16 * w + 15, last) / a.H;  // this wave's last position
  const int wmin = first_key(a, pos0 + min(r0 + 16 * w, last) / a.H);  // and first key
  const int fp = __builtin_amdgcn_readfirstlane(first_key(a, pos0 + r0 / a.H) / PAGE);
  const int npages = __builtin_amdgcn_readfirstlane((pos0 + last / a.H) / PAGE + 1);
  const int pps = __builtin_amdgcn_readfirstlane((npages - fp + a.nsplit - 1) / a.nsplit);
  const int p0 = fp + blockIdx.y * pps, p1 = min(p0 + pps, npages);
  const int* bt = a.bt + (long)b * a.W;
  const unsigned short* cache = (const unsigned short*)a.cache;
  const long nrows = (long)a.Nt * a.H;

  if (p0 >= p1) {  // an empty split: only reachable with nsplit > 1
    if (myrow <= last && g == 0) {
      float* ml = a.part_ml + 2 * (blockIdx.y * nrows + base + myrow);
      ml[0] = NEG;
      ml[1] = 0.f;
    }
    return;
  }

  bf16x8 qf[G::KT];
  {
    const bf16x8* qp = (const bf16x8*)((const unsigned short*)a.q + (base + row) * G::QP + 8 * g);
#pragma unroll
    for (int k = 0; k < G::KT; ++k) qf[k] = qp[4 * k];
  }

  int ids = 0;  // lane j: the id of page pb + j
  int pb = p0 - 64;
  const int per = 2 * G::KT / nw;  // DMA instructions per page and wave, rounded down
  auto dma = [&](int p) {
    if (p - pb >= 64) {
      pb = p;
      ids = bt[min(p + lane, p1 - 1)];
    }
    const int page = __builtin_amdgcn_readlane(ids, p - pb);
    page_dma<G>(cache + (long)page * PAGE * G::QP, smem + (p - p0) % G::NB * G::PAGEB, w, nw, lane);
  };
  for (int p = p0; p < min(p0 + G::NB - 1, p1); ++p) dma(p);
  const unsigned lds0 = (unsigned)(uintptr_t)(KGS_LDS char*)smem;
  unsigned ka[G::NP], va[G::NP][2];
#pragma unroll
  for (int k = 0; k < G::NP; ++k) {
    ka[k] = lds0 + G::off(l16, 4 * k + g);
#pragma unroll
    for (int x = 0; x < 2; ++x) va[k][x] = lds0 + G::off(4 * g + tq, 2 * (2 * k + x) + (tp >> 1)) + 8 * (tp & 1);
  }

  f32x4 acc[2 * RT];
#pragma unroll
  for (int i = 0; i < 2 * RT; ++i) acc[i] = f32x4{};
  float m = NEG, l = 0.f;
  const float sl2 = a.sl2;

  for (int p = p0; p < p1; ++p) {
    vm_wait(min(G::NB - 2, p1 - 1 - p) * per);
    asm volatile("s_barrier" ::: "memory");
    if (p + G::NB - 1 < p1) dma(p + G::NB - 1);
    if (p * PAGE <= wmax && p * PAGE + PAGE > wmin) {
      const unsigned slot = (p - p0) % G::NB * G::PAGEB;
      unsigned kp[G::NP], vp[G::NP][2];
#pragma unroll
      for (int k = 0; k < G::NP; ++k) {
        kp[k] = ka[k] + slot;
        vp[k][0] = va[k][0] + slot;
        vp[k][1] = va[k][1] + slot;
      }
      constexpr int KT = G::KT, KD = KT < 5 ? KT : 5;  // batches in flight
      KeyBatch kb[KD];
      f32x4 s2[2][2] = {};  // even and odd steps: two chains per key tile
      static_for<0, KD - 1>([&](auto kc) {
        constexpr int k = decltype(kc)::value;
        kb[k].template read<G, k>(kp[k % G::NP]);
      });
      static_for<0, KT>([&](auto kc) {
        constexpr int k = decltype(kc)::value;
        if constexpr (k + KD - 1 < KT) kb[(k + KD - 1) % KD].template read<G, k + KD - 1>(kp[(k + KD - 1) % G::NP]);
        constexpr int newer = (k + KD - 1 < KT ? KD - 1 : KT - 1 - k) * 2;
        kb[k % KD].template wait<newer>();
#pragma unroll
        for (int t = 0; t < 2; ++t)
          s2[t][k & 1] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kb[k % KD].f[t], qf[k], s2[t][k & 1], 0, 0, 0);
      });
      f32x4 s[2] = {s2[0][0] + s2[0][1], s2[1][0] + s2[1][1]};
      float mx = m;
#pragma unroll
      for (int t = 0; t < 2; ++t)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int key = p * PAGE + 16 * t + 4 * g + r;
          if (key > pos || key < lo) s[t][r] = NEG;
          mx = fmaxf(mx, s[t][r]);
        }
      mx = xor32_max(xor16_max(mx));
      const bool grow = (mx - m) * sl2 > RESCALE;
      if (__any(grow)) {
        const float mn = grow ? mx : m;
        const float alpha = __builtin_amdgcn_exp2f((m - mn) * sl2);
        m = mn;
        l *= alpha;
#pragma unroll
        for (int i = 0; i < 2 * RT; ++i) acc[i] *= alpha;
      }
      const float msl = m * sl2;
      float pr[8];
#pragma unroll
      for (int t = 0; t < 2; ++t)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const float e = s[t][r] == NEG ? 0.f : __builtin_amdgcn_exp2f(__builtin_fmaf(s[t][r], sl2, -msl));
          pr[4 * t + r] = e;
          l += e;
        }
      // the first C^T fragments are on their way under the packing of P
      constexpr int PD = RT < 4 ? RT : 4;
      TrBatch v[PD];
      static_for<0, PD - 1>([&](auto jc) {
        constexpr int j = decltype(jc)::value;
        v[j].template read<G, j>(vp[j % G::NP]);
      });
      const bf16x8 pf = pack_bf16x8(pr, 0);
      static_for<0, RT>([&](auto jc) {
        constexpr int j = decltype(jc)::value;
        if constexpr (j + PD - 1 < RT) v[(j + PD - 1) % PD].template read<G, j + PD - 1>(vp[(j + PD - 1) % G::NP]);
        constexpr int newer = (j + PD - 1 < RT ? PD - 1 : RT - 1 - j) * 4;
        v[j % PD].template wait<newer>();
#pragma unroll
        for (int x = 0; x < 2; ++x)
          acc[2 * j + x] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v[j % PD].frag(x), pf, acc[2 * j + x], 0, 0, 0);
      });
    }
  }
  l = xor32_sum(xor16_sum(l));
  if (myrow > last) return;
  if (a.nsplit == 1) {
    const float inv = 1.0f / l;
    unsigned short* op = (unsigned short*)a.o + (base + myrow) * G::RP + 4 * g;
#pragma unroll
    for (int i = 0; i < 2 * RT; ++i) {
      uint2 v;
      v.x = pack_bf16x2(acc[i][0] * inv, acc[i][1] * inv);
      v.y = pack_bf16x2(acc[i][2] * inv, acc[i][3] * inv);
      *(uint2*)(op + 16 * i) = v;
    }
  } else {
    const long pr = blockIdx.y * nrows + base + myrow;
    float* po = a.part_o + pr * G::RP + 4 * g;
#pragma unroll
    for (int i = 0; i < 2 * RT; ++i) *(f32x4*)(po + 16 * i) = acc[i];
    if (g == 0) {
      a.part_ml[2 * pr] = m;
      a.part_ml[2 * pr + 1] = l;
    }
  }
}

// one workgroup per row: o = sum_s 2^((m_s - m) sl2) acc_s / sum_s 2^((m_s - m) sl2) l_s
constexpr int MAX_SPLIT = 64;
__global__ __launch_bounds__(128) void merge(Args a) {
  __shared__ float wt[MAX_SPLIT];
  const int tid = threadIdx.x;
  const long nrows = (long)a.Nt * a.H, row = blockIdx.x;
  if (tid < 64) {
    float m = NEG, l = 0.f;
    if (tid < a.nsplit) {
      const float* ml = a.part_ml + 2 * (tid * nrows + row);
      l = ml[1];
      m = l > 0.f ? ml[0] : NEG;
    }
    const float mx = wave_max(m);
    const float e = l > 0.f ? __builtin_amdgcn_exp2f((m - mx) * a.sl2) : 0.f;
    wt[tid] = e / wave_sum(e * l);
  }
  __syncthreads();
  for (int c = 4 * tid; c < a.RP; c += 512) {
    f32x4 v = f32x4{};
#pragma unroll 4
    for (int s = 0; s < a.nsplit; ++s) {
      const float w = wt[s];
      if (w > 0.f) v += *(const f32x4*)(a.part_o + (s * nrows + row) * a.RP + c) * w;
    }
    uint2 o;
    o.x = pack_bf16x2(v[0], v[1]);
    o.y = pack_bf16x2(v[2], v[3]);
    *(uint2*)((unsigned short*)a.o + row * a.RP + c) = o;
  }
}

// ---------------------------------------------------------------- attn_simple
constexpr int SIMPLE_MAX = 2048;  // largest RP
constexpr int SIMPLE_ROT = 512;   // and HR

template <typename T>
__global__ __launch_bounds__(256) void attn_simple(Args a) {
  __shared__ float qs[SIMPLE_MAX + SIMPLE_ROT];
  __shared__ float ps[256];
  __shared__ float red[4];
  const int tid = threadIdx.x, RP = a.RP, QP = RP + a.HR;
  const long row = blockIdx.x;
  const int tok = (int)(row / a.H), pos = a.tok_pos[tok], lo = first_key(a, pos);
  const int* bt = a.bt + (long)a.tok_seq[tok] * a.W;
  const T* cache = (const T*)a.cache;
  for (int i = tid; i < QP; i += 256) qs[i] = ld((const T*)a.q + row * QP + i);
  float acc[SIMPLE_MAX / 256];
#pragma unroll
  for (int i = 0; i < SIMPLE_MAX / 256; ++i) acc[i] = 0.f;
  float m = NEG, l = 0.f;
  __syncthreads();
  for (int k0 = lo; k0 <= pos; k0 += 256) {
    const int key = k0 + tid;
    float s = NEG;
    if (key <= pos) {
      const T* c = cache + ((long)bt[key / PAGE] * PAGE + key % PAGE) * QP;
      s = 0.f;
      for (int i = 0; i < QP; ++i) s = __builtin_fmaf(qs[i], ld(c + i), s);
      s *= a.scale;
    }
    float mx = wave_max(s);
    if ((tid & 63) == 0) red[tid >> 6] = mx;
    __syncthreads();
    mx = fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3]));
    mx = fmaxf(mx, m);
    const float e = key <= pos ? expf(s - mx) : 0.f;
    ps[tid] = e;
    const float alpha = expf(m - mx);
    m = mx;
    const float sum = wave_sum(e);
    __syncthreads();
    if ((tid & 63) == 0) red[tid >> 6] = sum;
    __syncthreads();
    l = l * alpha + (red[0] + red[1] + red[2] + red[3]);
    const int nk = min(256, pos + 1 - k0);
#pragma unroll
    for (int i = 0; i < SIMPLE_MAX / 256; ++i) {
      const int col = tid + 256 * i;
      if (col < RP) {
        float v = acc[i] * alpha;
        for (int j = 0; j < nk; ++j) {
          const int kj = k0 + j;
          v = __builtin_fmaf(ps[j], ld(cache + ((long)bt[kj / PAGE] * PAGE + kj % PAGE) * QP + col), v);
        }
        acc[i] = v;
      }
    }
    __syncthreads();
  }
  const float inv = 1.0f / l;
#pragma unroll
  for (int i = 0; i < SIMPLE_MAX / 256; ++i) {
    const int col = tid + 256 * i;
    if (col < RP) st((T*)a.o + row * RP + col, acc[i] * inv);
  }
}

template <int RT, int RK>
static hipError_t launch_attn(const Args& a, int ntiles, int nw, hipStream_t s) {
  const size_t lds = Geo<RT, RK>::NB * Geo<RT, RK>::PAGEB;
  if (lds > 48 * 1024) {
    const hipError_t e =
        hipFuncSetAttribute((const void*)attn<RT, RK>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    if (e != hipSuccess) return e;
  }
  hipLaunchKernelGGL((attn<RT, RK>), dim3(ntiles, a.nsplit), dim3(64 * nw), lds, s, a);
  return hipGetLastError();
}
template <int RT>
static hipError_t launch_attn(const Args& a, int ntiles, int nw, hipStream_t s) {
  return a.HR == 0 ? launch_attn<RT, 0>(a, ntiles, nw, s)
                   : a.HR == 32 ? launch_attn<RT, 1>(a, ntiles, nw, s) : launch_attn<RT, 2>(a, ntiles, nw, s);
}

}  // namespace latent
}  // namespace kgs

// hr: columns of the rotated key part from okr on (0: none), which go after the rp of the
// latent, turned by pos with cs [npos][rot / 2][cos, sin] (neighbouring pairs)
KGS_EXPORT int kgs_latent_norm(const void* z, long ldz, int oq, int nq, int qp, int oc, int nc, int rp, int okr, int hr,
                               const void* cs, const void* pos, int npos, int rot, const void* wq, const void* wc,
                               void* cq, void* cache, const void* slots, int T, float eps, int f32, hipStream_t s) {
  using namespace kgs::latent;
  if (T <= 0 || nq <= 0 || qp < nq || nc < 0 || (nc && rp < nc) || oq < 0 || oc < 0 || ldz < oq + nq ||
      (nc && ldz < oc + nc) || hr < 0)
    return KGS_ERR_SHAPE;
  if (hr && (!nc || !cs || !pos || npos <= 0 || rot <= 0 || rot > hr || (rot | hr) % 8 || okr < 0 || ldz < okr + hr))
    return KGS_ERR_SHAPE;
  NormArgs a{z, ldz, oq, nq, qp, oc, nc, rp, okr, hr, (const float*)cs, (const int*)pos, npos, rot,
             (const float*)wq, (const float*)wc, cq, cache, (const int*)slots, eps};
  const bool vec = !f32 && ((nq | qp | nc | rp | oq | oc | okr) & 7) == 0 && hr <= 512 && ldz % 8 == 0 && qp <= 512 * NORM_NV &&
                   (!nc || rp <= 512 * NORM_NV) && (((uintptr_t)z | (uintptr_t)cq | (uintptr_t)cache | (uintptr_t)wq | (uintptr_t)wc) & 15) == 0;
  if (vec) hipLaunchKernelGGL(norm_vec, dim3((T + 3) / 4, nc ? 2 : 1), dim3(256), 0, s, a, T);
  else if (f32) hipLaunchKernelGGL(norm<float>, dim3(T, nc ? 2 : 1), dim3(256), 0, s, a);
  else hipLaunchKernelGGL(norm<unsigned short>, dim3(T, nc ? 2 : 1), dim3(256), 0, s, a);
  return (int)hipGetLastError();
}

// out[out_row(i)][h][n] = (sum_k a[in_row(i)][h][k] w[h][n][k]) * sigmoid(gate[out_row(i)][h hg + n eg]);
// hr more columns of a, after the K, go after the N of out, turned by pos[i] (cs as above)
KGS_EXPORT int kgs_head_proj(const void* a, const void* w, void* out, const void* idx_in, const void* idx_out,
                             const void* gate, long lda, long ha, long ldo, long ho, long ldg, int hg, int eg, int Nt,
                             int H, int N, int K, int hr, const void* cs, const void* pos, int npos, int rot, int f32,
                             hipStream_t s) {
  using namespace kgs::latent;
  if (Nt <= 0 || H <= 0 || N <= 0 || K <= 0 || hr < 0 || ha < K + hr || ho < N + hr || lda < (H - 1) * ha + K + hr ||
      ldo < (H - 1) * ho + N + hr || H > 65535)
    return KGS_ERR_SHAPE;
  if (hr && (hr % 16 || !cs || !pos || npos <= 0 || rot <= 0 || rot > hr || rot % 8)) return KGS_ERR_SHAPE;
  if (gate && (hg < 1 || eg < 0 || eg > 1 || ldg < (long)(H - 1) * hg + (eg ? N : 1))) return KGS_ERR_SHAPE;
  ProjArgs p{a, w, out, (const int*)idx_in, (const int*)idx_out, gate, lda, ha, ldo, ho, ldg, hg, eg, Nt, H, N, K,
             hr, npos, rot, (const float*)cs, (const int*)pos};
  if (f32) {
    hipLaunchKernelGGL(head_proj_f32, dim3(Nt, H), dim3(256), 0, s, p);
    return (int)hipGetLastError();
  }
  if (N % 16 || K % 32) return KGS_ERR_SHAPE;
  if ((((uintptr_t)a | (uintptr_t)w | (uintptr_t)out) & 15) || (lda | ha) % 8 || (ldo | ho) % 4) return KGS_ERR_ALIGN;
  const int gx = ((N + hr) / 16 + 3) / 4;
  if (Nt <= 16) hipLaunchKernelGGL(head_proj<1>, dim3(gx, 1, H), dim3(256), 0, s, p);
  else if (Nt <= 32) hipLaunchKernelGGL(head_proj<2>, dim3(gx, 1, H), dim3(256), 0, s, p);
  else if ((Nt + 63) / 64 > 65535) return KGS_ERR_SHAPE;
  else hipLaunchKernelGGL(head_proj<4>, dim3(gx, (Nt + 63) / 64, H), dim3(256), 0, s, p);
  return (int)hipGetLastError();
}

// MFMA form: RP one of 32 x {1, 2, 3, 4, 6, 8, 12, 16}, HR 0, 32 or 64, bf16. ntiles workgroups
// per split (items: ntiles (sequence, tile) pairs; null: B x tiles). A tile is
// 16 nw rows.
KGS_EXPORT int kgs_latent_attn(const void* q, const void* cache, void* o, void* part_o, void* part_ml, const void* q0,
                               const void* n, const void* pos0, const void* bt, const void* items, int ntiles,
                               int tiles, int nw, int nsplit, int H, int W, int Nt, int RP, int HR, int win,
                               float scale, hipStream_t s) {
  using namespace kgs::latent;
  if (ntiles <= 0 || H <= 0 || W <= 0 || Nt <= 0 || nw < 1 || nw > 8 || nsplit < 1 || nsplit > MAX_SPLIT ||
      (!items && tiles <= 0) || (HR != 0 && HR != 32 && HR != 64) || win < 0)
    return KGS_ERR_SHAPE;
  if (nsplit > 1 && (!part_o || !part_ml)) return KGS_ERR_ARG;
  if (RP > 256 && nw > 4) return KGS_ERR_SHAPE;  // a wave holds 16 x RP outputs in registers
  if (((uintptr_t)q | (uintptr_t)cache | (uintptr_t)o | (uintptr_t)part_o) & 15) return KGS_ERR_ALIGN;
  Args a{q, cache, o, (float*)part_o, (float*)part_ml, (const int*)q0, (const int*)n, (const int*)pos0,
         (const int*)bt, (const int*)items, nullptr, nullptr, H, W, tiles, nsplit, Nt, RP, HR, scale,
         scale * 1.4426950408889634f, win};
  hipError_t e;
  switch (RP) {
    case 32: e = launch_attn<1>(a, ntiles, nw, s); break;
    case 64: e = launch_attn<2>(a, ntiles, nw, s); break;
    case 96: e = launch_attn<3>(a, ntiles, nw, s); break;
    case 128: e = launch_attn<4>(a, ntiles, nw, s); break;
    case 192: e = launch_attn<6>(a, ntiles, nw, s); break;
    case 256: e = launch_attn<8>(a, ntiles, nw, s); break;
    case 384: e = launch_attn<12>(a, ntiles, nw, s); break;
    case 512: e = launch_attn<16>(a, ntiles, nw, s); break;
    default: return KGS_ERR_SHAPE;
  }
  if (e == hipSuccess && nsplit > 1) {
    hipLaunchKernelGGL(merge, dim3((unsigned)((long)Nt * H)), dim3(128), 0, s, a);
    e = hipGetLastError();
  }
  return (int)e;
}

KGS_EXPORT int kgs_latent_attn_simple(const void* q, const void* cache, void* o, const void* tok_seq,
                                      const void* tok_pos, const void* bt, int H, int W, int Nt, int RP, int HR, int win,
                                      float scale, int f32, hipStream_t s) {
  using namespace kgs::latent;
  if (H <= 0 || W <= 0 || Nt <= 0 || RP <= 0 || RP > SIMPLE_MAX || HR < 0 || HR > SIMPLE_ROT || win < 0)
    return KGS_ERR_SHAPE;
  Args a{q, cache, o, nullptr, nullptr, nullptr, nullptr, nullptr, (const int*)bt, nullptr, (const int*)tok_seq,
         (const int*)tok_pos, H, W, 0, 1, Nt, RP, HR, scale, 0.f, win};
  const dim3 grid((unsigned)((long)Nt * H));
  if (f32) hipLaunchKernelGGL(attn_simple<float>, grid, dim3(256), 0, s, a);
  else hipLaunchKernelGGL(attn_simple<unsigned short>, grid, dim3(256), 0, s, a);
  return (int)hipGetLastError();
}
