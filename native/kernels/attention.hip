// Flash-attention forward for gfx950 (bf16 in/out, fp32 softmax/accumulate),
// head_dim 128, causal or full, GQA -- the prefill attention of the Llama
// stand-in (kgs/models/llama.py); and its ragged form (head_dim 64 or 128, prompt
// portions of any length at any position, an optional output gate, window, and a further
// part of the keys that all heads share and that turns with the position) for
// latent attention over expanded keys and values. Q, K and V are read in place from the fused
// QKV projection output ([tokens, (H + 2 HKV) * 128], any row stride) and O is
// written as [tokens, H * 128], the layout the O projection consumes: no
// transposes around the kernel.
//
// Structure (one workgroup = 4 waves = 128 query rows of one (batch, head);
// 2 workgroups per CU; K/V tiles of 64 keys):
//   * swapped QK^T on v_mfma_f32_32x32x16_bf16: S^T = K . Q^T, so a lane owns
//     ONE query row (lane & 31) and 32 of the tile's 64 scores -- the row max /
//     row sum are in-lane plus one xor-32 exchange, and the per-row rescale of
//     O is a lane scalar;
//   * the S^T accumulator is the B operand of P.V with no data movement
//     (O^T = V^T . P^T): registers 8s..8s+7 of each 32x32 tile are k-step s,
//     in the permuted key order kv = 16s + 8(j>>2) + 4(lane>>5) + (j&3) that
//     the V fragments are read in;
//   * V fragments via ds_read_b64_tr_b16 (a free transpose out of the
//     row-major tile), K fragments via ds_read_b128; both tiles use the
//     256-B-row XOR image off(r, c) = 256 r + 16 (c ^ ((r&3)<<2 | (r>>2)&3)),
//     conflict-free for the 16-lane groups of ds_read_b128 and the 32-lane
//     halves of the transposed read;
//   * double buffer filled by LDS-DMA: the next K/V tile's global_load_lds
//     are issued before the current tile's MFMAs (no staging registers),
//     vmcnt(0) + one barrier per tile;
//   * causal: fully-masked tiles are skipped per wave, the diagonal tiles are
//     masked in registers; q-blocks are dispatched heaviest first, and the four
//     query heads sharing a KV head are dealt to the same XCD back to back so
//     the K/V tiles they share are L2 hits.
#include "kgs_common.h"

namespace kgs {
namespace attn {

typedef float f32x16 __attribute__((ext_vector_type(16)));

constexpr int QB = 128;  // query rows per workgroup (4 waves x 32)
constexpr int KB = 64;   // keys per tile
constexpr float NEG = -1.0e30f;
constexpr float RESCALE = 8.0f;  // deferred-max threshold, log2 units: P <= 256

struct Args {
  const unsigned short* q;
  const unsigned short* k;
  const unsigned short* v;
  unsigned short* o;
  long ldq, ldk, ldv, ldo;  // row strides (elements)
  int B, S, H, HKV;
  float sl2;  // softmax scale * log2(e)
  int causal;
  int Sk;    // keys per sequence (= S, or S + qoff for a chunk over a cached context)
  int qoff;  // position of query row 0 among the keys: causal row i sees keys <= qoff + i
  // ragged form: one int4 per (sequence, q-block) -- first query row, first key
  // row of the sequence, position of the first query row, valid query rows
  const int4* items;
  // or null: [rows, ldg], element n of head h's output times sigmoid(gate[row][h hg + n eg])
  const unsigned short* gate;
  long ldg;
  int hg, eg;
  const unsigned short* kr;  // rotated key part: [key rows, ldr], HR columns, already turned
  long ldr;
  // q's part of it follows each head's HD columns and is turned on load: by the row's
  // position, neighbouring pairs, cs [npos][rot] (cos, sin)
  const float* cs;
  const int* pos;
  int npos, rot;
  int win;  // a row sees itself and the win - 1 keys before it; 0: all
};

// XOR image of a row's 16-B chunks (HD / 8 of them)
template <int HD>
__device__ __forceinline__ int swz(int r) {
  if constexpr (HD == 128) return ((r & 3) << 2) | ((r >> 2) & 3);
  if constexpr (HD == 32) return (r >> 2) & 3;
  return ((r & 2) << 1) | ((r >> 2) & 3);
}
template <int HD>
__device__ __forceinline__ int off(int r, int c) { return 2 * HD * r + 16 * (c ^ swz<HD>(r)); }

__device__ __forceinline__ bf16x8 pack8(const f32x16& s, int base) { return pack_bf16x8(s, base); }

// RAGGED: any number of query rows per sequence at any position (Args::items),
// rows and keys past a block's end clamped on load and dropped on store; always
// causal. Otherwise B equal sequences of S rows, a multiple of QB.
template <int HD, bool RAGGED, int HR = 0>
__global__ __launch_bounds__(256, 2) __attribute__((amdgpu_waves_per_eu(2, 2))) void fwd(Args a) {
  constexpr int TILE_BYTES = KB * HD * 2;  // 16 KB at 128
  constexpr int ND = HD / 32, NK = HD / 16, NR = HR / 16, ROT_BYTES = KB * HR * 2;
  __shared__ __attribute__((aligned(16))) char smem[2][2 * TILE_BYTES + ROT_BYTES];  // [buf]: K, V, rotated K

  const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int l32 = lane & 31, hh = lane >> 5;
  int h, kvh, q0, qw, qrow, qoff, nval = QB;
  long tok0, ktok0;
  bool causal = true;
  if constexpr (RAGGED) {
    const int item = blockIdx.x / a.H;
    h = kvh = blockIdx.x - item * a.H;
    const int4 it = a.items[item];
    tok0 = it.x;
    ktok0 = it.y;
    qoff = it.z;
    nval = it.w;
    q0 = 0;
    qw = 32 * w;
    qrow = qw + l32;
  } else {
    const int nqb = a.S / QB;
    const int nwg = gridDim.x;
    // XCD-aware order: 8 consecutive dispatch slots of one XCD take 4 heads of
    // one KV group; work ids stay heaviest-first in dispatch time.
    int lid = blockIdx.x;
    if ((nwg & 31) == 0) {
      const int t = lid >> 3, x = lid & 7;
      lid = ((t >> 2) << 5) | (x << 2) | (t & 3);
    }
    const int per = a.B * a.H;
    const int qi = lid / per, rem = lid - qi * per;
    const int qb = a.causal ? nqb - 1 - qi : qi;
    const int b = rem / a.H;
    h = rem - b * a.H;
    kvh = h / (a.H / a.HKV);

    q0 = qb * QB;
    qw = q0 + 32 * w;       // this wave's first query row
    qrow = qw + l32;        // this lane's query row
    tok0 = (long)b * a.S;     // first query token of the sequence
    ktok0 = (long)b * a.Sk;   // its first key token
    qoff = a.qoff;
    causal = a.causal != 0;
  }
  const int lrow = RAGGED ? min(qrow, nval - 1) : qrow;  // the row this lane loads

  // Q fragments (B operand of S^T = K.Q^T): lane holds Q[qrow][16ks + 8hh .. +7]
  bf16x8 qf[NK + NR];
  {
    const bf16x8* qp = (const bf16x8*)(a.q + (tok0 + lrow) * a.ldq + (long)h * (HD + HR) + 8 * hh);
#pragma unroll
    for (int ks = 0; ks < NK + NR; ++ks) qf[ks] = qp[2 * ks];
    if constexpr (HR > 0) {
      const float* cs = a.cs + (long)min(max(a.pos[tok0 + lrow], 0), a.npos - 1) * a.rot + 8 * hh;
#pragma unroll
      for (int ks = 0; ks < NR; ++ks)
        if (16 * ks + 8 * hh < a.rot) {
          float y[8];
#pragma unroll
          for (int i = 0; i < 8; i += 2) {
            const float u = bf2f((unsigned short)qf[NK + ks][i]), v = bf2f((unsigned short)qf[NK + ks][i + 1]);
            y[i] = rope_lo(u, v, cs[16 * ks + i], cs[16 * ks + i + 1]);
            y[i + 1] = rope_hi(u, v, cs[16 * ks + i], cs[16 * ks + i + 1]);
          }
          qf[NK + ks] = pack_bf16x8(y, 0);
        }
    }
  }

  const unsigned short* kbase = a.k + ktok0 * a.ldk + (long)kvh * HD;
  const unsigned short* vbase = a.v + ktok0 * a.ldv + (long)kvh * HD;
  const unsigned short* rbase = a.kr + ktok0 * a.ldr;
  // K/V tile jn -> LDS buffer sb by LDS-DMA (global_load_lds, no staging
  // registers): a 16 KB tile is 16 chunks of 1 KB = 4 rows of 256 B; wave w
  // issues chunks 4w .. 4w+3 of K and of V. Lane l lands at chunk + 16 l, i.e.
  // at slot (r, c') of the XOR image, so it fetches column c = c' ^ swz(r).
  auto dma_tiles = [&](int jn, int sb) {
    int lane = threadIdx.x & 63;
    if constexpr (HD + HR >= 160) asm volatile("" : "+v"(lane));  // offsets made anew: hoisted they would spill
#pragma unroll
    for (int i = 0; i < ND; ++i) {
      const int ch = ND * w + i;
      const int r = (512 / HD) * ch + lane / (HD / 8), c = (lane & (HD / 8 - 1)) ^ swz<HD>(r);
      long row = (long)jn * KB + r;
      if constexpr (RAGGED) row = min(row, (long)(qoff + nval - 1));
      glds16(kbase + row * a.ldk + 8 * c, smem[sb] + 1024 * ch);
      glds16(vbase + row * a.ldv + 8 * c, smem[sb] + TILE_BYTES + 1024 * ch);
    }
    if constexpr (HR > 0) {
#pragma unroll
      for (int i = 0; i < HR / 32; ++i) {
        const int ch = HR / 32 * w + i;
        const int r = (512 / HR) * ch + lane / (HR / 8), c = (lane & (HR / 8 - 1)) ^ swz<HR>(r);
        const long row = min((long)jn * KB + r, (long)(qoff + nval - 1));
        glds16(rbase + row * a.ldr + 8 * c, smem[sb] + 2 * TILE_BYTES + 1024 * ch);
      }
    }
  };

  const int ntile = RAGGED ? (qoff + nval - 1) / KB + 1 : causal ? (qoff + q0 + QB) / KB : a.Sk / KB;
  const int win = RAGGED ? a.win : 0;
  const int j0 = win ? max(0, qoff + q0 - win + 1) / KB : 0;
  dma_tiles(j0, 0);
  // Q fragments and tile 0 complete before the loop (a vmcnt the waitcnt pass
  // sees, so it does not carry the Q loads into the loop header)
  __builtin_amdgcn_s_waitcnt(0x0f70);  // vmcnt(0)
  __syncthreads();

  f32x16 o[ND];
#pragma unroll
  for (int d = 0; d < ND; ++d) o[d] = f32x16{};
  float m = NEG, l = 0.f;
  const float sl2 = a.sl2;

  // tr-read lane address pieces: group g = lane >> 4, lane 4q + p in it
  int g = lane >> 4, tq = (lane >> 2) & 3, tp = lane & 3;

  for (int j = j0; j < ntile; ++j) {
    const int buf = (j - j0) & 1;
    // the other buffer was released by the previous tile's barrier
    if (j + 1 < ntile) dma_tiles(j + 1, buf ^ 1);
    const int kv0 = j * KB;
    if constexpr (HD + HR >= 160) asm volatile("" : "+v"(tq), "+v"(g));  // V addresses made anew: hoisted they would spill
    if ((!causal || kv0 <= qoff + qw + 31) && (!win || kv0 + KB > qoff + qw - win + 1)) {
      const char* Ks = smem[buf];
      const char* Vs = smem[buf] + TILE_BYTES;
      f32x16 s[2];
      if constexpr (HR == 0) {
        // all 16 K fragments of the tile are read up front (the registers the
        // LDS-DMA staging freed), so the QK^T MFMAs never wait on one LDS read
        bf16x8 kf[2][NK];
#pragma unroll
        for (int t = 0; t < 2; ++t)
#pragma unroll
          for (int ks = 0; ks < NK; ++ks) kf[t][ks] = *(const bf16x8*)(Ks + off<HD>(32 * t + l32, 2 * ks + hh));
        __builtin_amdgcn_sched_barrier(0);  // keep the reads ahead (the scheduler sinks them otherwise)
#pragma unroll
        for (int t = 0; t < 2; ++t) {
          s[t] = f32x16{};
#pragma unroll
          for (int ks = 0; ks < NK; ++ks) s[t] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(kf[t][ks], qf[ks], s[t], 0, 0, 0);
        }
      } else {
        // 32 keys at a time: with the rotated part all fragments at once do not fit
#pragma unroll
        for (int t = 0; t < 2; ++t) {
          bf16x8 kf[NK + NR];
#pragma unroll
          for (int ks = 0; ks < NK; ++ks) kf[ks] = *(const bf16x8*)(Ks + off<HD>(32 * t + l32, 2 * ks + hh));
#pragma unroll
          for (int ks = 0; ks < NR; ++ks)
            kf[NK + ks] = *(const bf16x8*)(Ks + 2 * TILE_BYTES + off<HR>(32 * t + l32, 2 * ks + hh));
          if (t == 0) __builtin_amdgcn_sched_barrier(0);
          s[t] = f32x16{};
#pragma unroll
          for (int ks = 0; ks < NK + NR; ++ks) s[t] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(kf[ks], qf[ks], s[t], 0, 0, 0);
        }
      }
      // the first half of the tile's V fragments is read now, so its LDS
      // latency hides under the softmax below (all 16 would spill at 2 waves
      // per SIMD); the second half is read under the first half's P.V MFMAs
      bf16x8 vfr[ND][2][2];
      auto read_v = [&](int d) {
        const int c0 = 4 * d + 2 * (g & 1) + (tp >> 1);
#pragma unroll
        for (int t = 0; t < 2; ++t)
#pragma unroll
          for (int sp = 0; sp < 2; ++sp) {
            const int kvb = 32 * t + 16 * sp + 4 * hh + tq;
            vfr[d][t][sp] = tr_frag(Vs + off<HD>(kvb, c0) + 8 * (tp & 1), Vs + off<HD>(kvb + 8, c0) + 8 * (tp & 1));
          }
      };
      read_v(0);
      if constexpr (HD + HR < 160) read_v(1);  // registers
      __builtin_amdgcn_sched_barrier(0);
      if ((causal && kv0 + KB - 1 > qoff + qw) || (win && kv0 < qoff + qw + 31 - win + 1)) {
        const int lo = win ? qoff + qrow - win + 1 : 0;
#pragma unroll
        for (int t = 0; t < 2; ++t)
#pragma unroll
          for (int r = 0; r < 16; ++r) {
            const int kv = kv0 + 32 * t + (r & 3) + 8 * (r >> 2) + 4 * hh;
            if (kv > qoff + qrow || (RAGGED && kv < lo)) s[t][r] = NEG;
          }
      }
      float mx = m;
#pragma unroll
      for (int t = 0; t < 2; ++t)
#pragma unroll
        for (int r = 0; r < 16; ++r) mx = fmaxf(mx, s[t][r]);
      mx = xor32_max(mx);  // v_permlane32_swap (kgs_common.h), not an LDS round trip
      // deferred rescale (guide T13): the running max m only moves when a row's
      // new max exceeds it by more than RESCALE (log2 units after sl2), so most
      // tiles skip the 64-multiply O rescale; p = exp2(s sl2 - m sl2) then stays
      // <= 2^RESCALE (fp32 sums and bf16 P are scale-free). Both l and O see the
      // same alpha, and the decision is wave-uniform, so no pending P.V is split.
      const bool grow = (mx - m) * sl2 > RESCALE;
      if (__any(grow)) {
        const float mn = grow ? mx : m;
        const float alpha = __builtin_amdgcn_exp2f((m - mn) * sl2);
        m = mn;
        l *= alpha;
#pragma unroll
        for (int d = 0; d < ND; ++d) o[d] *= alpha;
      }
      const float msl = RAGGED && m == NEG ? 0.f : m * sl2;  // a row that has seen no key yet: weights 0
#pragma unroll
      for (int t = 0; t < 2; ++t)
#pragma unroll
        for (int r = 0; r < 16; ++r) {
          const float p = __builtin_amdgcn_exp2f(__builtin_fmaf(s[t][r], sl2, -msl));
          s[t][r] = p;
          l += p;
        }
      bf16x8 pf[2][2];
#pragma unroll
      for (int t = 0; t < 2; ++t) {
        pf[t][0] = pack8(s[t], 0);
        pf[t][1] = pack8(s[t], 8);
      }
      if constexpr (HD + HR >= 160) read_v(1);
      if constexpr (ND == 4) {
        read_v(2);
        read_v(3);
      }
#pragma unroll
      for (int d = 0; d < ND; ++d)
#pragma unroll
        for (int t = 0; t < 2; ++t)
#pragma unroll
          for (int sp = 0; sp < 2; ++sp)
            o[d] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vfr[d][t][sp], pf[t][sp], o[d], 0, 0, 0);
    }
    __builtin_amdgcn_s_waitcnt(0x0f70);  // vmcnt(0): the next tile has landed
    __syncthreads();
  }

  l = xor32_sum(l);
  float inv = 1.0f / l;
  if constexpr (RAGGED) {
    if (qrow >= nval) return;
    if (a.gate && !a.eg) inv /= 1.0f + __expf(-bf2f(a.gate[(tok0 + qrow) * a.ldg + (long)h * a.hg]));
  }
  unsigned short* op = a.o + (tok0 + qrow) * a.ldo + (long)h * HD;
#pragma unroll
  for (int d = 0; d < ND; ++d)
#pragma unroll
    for (int r4 = 0; r4 < 4; ++r4) {
      const int dcol = 32 * d + 8 * r4 + 4 * hh;
      if constexpr (RAGGED)
        if (a.gate && a.eg) {
          const bf16x4 z = *(const bf16x4*)(a.gate + (tok0 + qrow) * a.ldg + (long)h * a.hg + dcol);
#pragma unroll
          for (int i = 0; i < 4; ++i) o[d][4 * r4 + i] /= 1.0f + __expf(-bf2f((unsigned short)z[i]));
        }
      uint2 pk;
      pk.x = pack_bf16x2(o[d][4 * r4 + 0] * inv, o[d][4 * r4 + 1] * inv);
      pk.y = pack_bf16x2(o[d][4 * r4 + 2] * inv, o[d][4 * r4 + 3] * inv);
      *(uint2*)(op + dcol) = pk;
    }
}

}  // namespace attn
}  // namespace kgs

// q/k/v/o point at head 0 of token 0 ([B*S, ld] token-major); heads of one
// token are contiguous 128-element blocks. Requires head_dim 128, S % 128 == 0,
// H % HKV == 0, 16-B aligned pointers and ld % 8 == 0.
//
// _ex: Sk keys per sequence ([B*Sk, ld] k/v), Sk >= S, Sk - S a multiple of 64:
// the S query rows are the LAST S positions of the sequence (a prefill chunk
// over Sk - S cached tokens), so causal row i sees keys 0 .. Sk - S + i.
KGS_EXPORT int kgs_attn_fwd_bf16_ex(const void* q, const void* k, const void* v, void* o, int B, int S, int Sk, int H,
                                   int HKV, int hd, long ldq, long ldk, long ldv, long ldo, float scale, int causal,
                                   hipStream_t s) {
  using namespace kgs::attn;
  constexpr int HD = 128;
  if (B <= 0 || S <= 0 || H <= 0 || HKV <= 0 || H % HKV) return KGS_ERR_SHAPE;
  if (hd != HD || S % QB || Sk < S || (Sk - S) % KB) return KGS_ERR_SHAPE;
  if (ldq < (long)H * HD || ldk < (long)HKV * HD || ldv < (long)HKV * HD || ldo < (long)H * HD) return KGS_ERR_SHAPE;
  const uintptr_t al = (uintptr_t)q | (uintptr_t)k | (uintptr_t)v | (uintptr_t)o;
  if ((al & 15) || (ldq | ldk | ldv | ldo) & 7) return KGS_ERR_ALIGN;
  const long nwg = (long)B * H * (S / QB);
  if (nwg > 0x7fffffff) return KGS_ERR_SHAPE;
  Args a{(const unsigned short*)q, (const unsigned short*)k, (const unsigned short*)v, (unsigned short*)o,
         ldq, ldk, ldv, ldo, B, S, H, HKV, scale * 1.4426950408889634f, causal ? 1 : 0, Sk, Sk - S,
         nullptr, nullptr, 0, 0, 0, nullptr, 0, nullptr, nullptr, 0, 0, 0};
  hipLaunchKernelGGL((fwd<HD, false>), dim3((unsigned)nwg), dim3(256), 0, s, a);
  return (int)hipGetLastError();
}

KGS_EXPORT int kgs_attn_fwd_bf16(const void* q, const void* k, const void* v, void* o, int B, int S, int H, int HKV,
                                int hd, long ldq, long ldk, long ldv, long ldo, float scale, int causal,
                                hipStream_t s) {
  return kgs_attn_fwd_bf16_ex(q, k, v, o, B, S, S, H, HKV, hd, ldq, ldk, ldv, ldo, scale, causal, s);
}

// Causal attention of ragged sequences, head_dim 64 or 128, as many key heads as
// query heads. items: nitems int4 (first query row, first key row of its
// sequence, number of that query row's own key, rows <= 128), any order (heaviest first
// keeps the tail short). Every row index an item names must lie in q / o, every
// key row first_key + number in k / v. win: each row sees its own key and the win - 1 before
// it (0: all). gate: head h's element n times sigmoid(gate[row][h hg + n eg]) (eg 0 or 1).
// kr (hr 32 or 64, or 0): a further part of every head's keys, [key rows, ldr]; q then has hr
// columns after each head's hd, turned by the row's pos with cs [npos][rot / 2][cos, sin].
KGS_EXPORT int kgs_attn_fwd_ragged_bf16(const void* q, const void* k, const void* v, void* o, const void* items,
                                       int nitems, int H, int hd, long ldq, long ldk, long ldv, long ldo, float scale,
                                       const void* gate, long ldg, int hg, int eg, const void* kr, long ldr, int hr,
                                       const void* cs, const void* pos, int npos, int rot, int win, hipStream_t s) {
  using namespace kgs::attn;
  if (nitems <= 0 || H <= 0 || (hd != 64 && hd != 128) || (hr != 0 && hr != 32 && hr != 64) || win < 0) return KGS_ERR_SHAPE;
  const long w = (long)H * hd;
  if (ldq < w + (long)H * hr || ldk < w || ldv < w || ldo < w) return KGS_ERR_SHAPE;
  if (gate && (hg < 1 || eg < 0 || eg > 1 || ldg < (long)(H - 1) * hg + (eg ? hd : 1))) return KGS_ERR_SHAPE;
  if (hr && (!kr || !cs || !pos || npos <= 0 || rot <= 0 || rot > hr || rot % 8 || ldr < hr)) return KGS_ERR_SHAPE;
  const uintptr_t al = (uintptr_t)q | (uintptr_t)k | (uintptr_t)v | (uintptr_t)o | (uintptr_t)items | (uintptr_t)kr | (uintptr_t)cs;
  if ((al & 15) || (ldq | ldk | ldv | ldo | ldr) & 7) return KGS_ERR_ALIGN;
  if (gate && eg && (((uintptr_t)gate & 7) || ldg % 4 || hg % 4)) return KGS_ERR_ALIGN;
  if ((long)nitems * H > 0x7fffffff) return KGS_ERR_SHAPE;
  Args a{(const unsigned short*)q, (const unsigned short*)k, (const unsigned short*)v, (unsigned short*)o,
         ldq, ldk, ldv, ldo, 0, 0, H, H, scale * 1.4426950408889634f, 1, 0, 0,
         (const int4*)items, (const unsigned short*)gate, ldg, hg, eg,
         (const unsigned short*)kr, ldr, (const float*)cs, (const int*)pos, npos, rot, win};
  const dim3 grid((unsigned)(nitems * H));
  auto fn = hd == 128 ? (hr == 0 ? fwd<128, true> : hr == 32 ? fwd<128, true, 32> : fwd<128, true, 64>)
                      : (hr == 0 ? fwd<64, true> : hr == 32 ? fwd<64, true, 32> : fwd<64, true, 64>);
  hipLaunchKernelGGL(fn, grid, dim3(256), 0, s, a);
  return (int)hipGetLastError();
}
