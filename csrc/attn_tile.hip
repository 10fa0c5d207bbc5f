// Causal softmax attention of bf16 prompt rows over a paged K/V cache with the keys and values of a step staged in LDS once for all
// waves of a workgroup; one map per head (optional score cap) or the two maps of a differential head:
//
//   one map:   s(i, j) = f(scale <q_i, k_j>),  f(s) = cap * tanh(s / cap) or s;     out = softmax(s) v * oscale * sigmoid(gate)
//   two maps:  s_m(i, j) = scale * temp(i) * <q_(i, m), k_(j, m)>,  a_m = softmax(s_m) v,  o = a_1 - lambda a_2,
//              out = o / sqrt(mean(o^2) + eps) * oscale * sigmoid(gate)             (the definitions of attn_diff.hip)
//
// K cache [blocks, G, BS, maps * dim], V cache key-contiguous [blocks, G, vdim, BS].
//
// A workgroup's four waves hold 32 queries each (two MFMA column groups of 16) of up to 4 heads of ONE kv group: every staged tile of 32
// keys serves 128 (query, head) columns.  A tile lies in LDS as the MFMA fragments themselves (64 lanes x 16 bytes, 1 KB): K rows
// in the key order of attn_sink.hip's S^T accumulators, so P^T needs no shuffle, and V rows straight from the key-contiguous
// cache, so neither operand needs a transposed or swizzled read and the LDS-DMA of a fragment is one instruction per wave.
// Fragments of tile t + 1 travel into the other buffer while tile t is computed; one barrier per tile.  The running maximum moves only
// when a score exceeds it by more than kDefer (base 2): until then weights are at most 2^kDefer, exact alike in bf16 and f32.
#include "common.h"
#include "kernels.h"
#include "attn_frag.h"

namespace {

constexpr float kNegBig = -1e30f;
constexpr float kDefer = 8.f;
constexpr float kLog2e = 1.4426950408889634f;
constexpr int kRows = 32;   // queries of a wave
constexpr int CG = 2;       // column groups of 16 of a wave

typedef void __attribute__((address_space(3))) * lds_void_ptr;

struct TileParams {
  const bf16_t* q;
  long qs;
  const bf16_t* kc;
  const bf16_t* vc;
  const int* bt;
  int bt_stride;
  int H, G, dim, vdim, BS, bs_shift;   // bs_shift: log2(BS), -1 when BS is no power of two
  int wh;                              // heads of a workgroup (1, 2, 4; divides H / G)
  float scale, cap, tcoef;
  int tevery;
  const float* lam;
  float eps, inv_nv, oscale;
  const bf16_t* gate;
  long gs;
  int gcol;
};

// maximum over the four lane groups (lanes l, l ^ 16, l ^ 32, l ^ 48), in registers
LK_DEVICE float max_groups(float v) {
  const auto a = __builtin_amdgcn_permlane16_swap(__float_as_uint(v), __float_as_uint(v), false, false);
  const unsigned a0 = a[0], a1 = a[1];
  v = fmaxf(__uint_as_float(a0), __uint_as_float(a1));
  const auto b = __builtin_amdgcn_permlane32_swap(__float_as_uint(v), __float_as_uint(v), false, false);
  const unsigned b0 = b[0], b1 = b[1];
  return fmaxf(__uint_as_float(b0), __uint_as_float(b1));
}

// one fragment: lane l's 16 bytes at src go to LDS byte off + 16 l (off wave-uniform).  As assembly: the compiler would wait for the
// transfer before the next LDS read of the OTHER buffer; the loop below waits for it itself, ahead of its barrier.
LK_DEVICE void dma16(unsigned off, const void* src) {
  asm volatile("s_mov_b32 m0, %0\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %1, off" ::"s"(off), "v"(src) : "memory", "m0");
}

template <int KP, int VP, int NM, bool CAP>
__global__ __launch_bounds__(256, (CG * NM * (VP / 16 + KP / 32) * 4 <= 160 ? 2 : 1)) void tile_attention_kernel(
    TileParams p, const int* __restrict__ cu_q, const int* __restrict__ ctx_lens, const int* __restrict__ tile_seq,
    const int* __restrict__ tile_q0, bf16_t* __restrict__ out, long os) {
  constexpr int KS = KP / 32, VT = VP / 16, NK = NM * 2 * KS, FR = NK + VT;
  extern __shared__ __attribute__((aligned(16))) bf16_t lds[];   // [2][FR][512]
  const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6), n16 = lane & 15, g = lane >> 4;
  const int rep = p.H / p.G, ngr = rep / p.wh, kvh = blockIdx.x / ngr;
  const int head = kvh * rep + (blockIdx.x % ngr) * p.wh + w % p.wh;
  const int b = tile_seq[blockIdx.y], q0 = tile_q0[blockIdx.y];
  const int qbeg = cu_q[b], qlen = cu_q[b + 1] - qbeg, ctx = ctx_lens[b], past = ctx - qlen;
  const int rows = kRows * (4 / p.wh);                       // queries of the workgroup
  const int qw = q0 + (w / p.wh) * kRows;                    // this wave's first query
  const int k1 = min(ctx, past + q0 + rows), ntile = (k1 + 31) / 32;
  const int wend = qw < qlen ? min(ctx, past + qw + kRows) : 0;   // keys this wave's columns see
  const int kdim = NM * p.dim;

  // queries past the sequence's end compute with its last row and are not stored
  uint4_t qf[CG][NM][KS];
  float hs[CG];
  int qpos[CG];
#pragma unroll
  for (int x = 0; x < CG; ++x) {
    const int qi = qw + 16 * x + n16;
    qpos[x] = past + qi;
    const bf16_t* qrow = p.q + (long)(qbeg + min(qi, qlen - 1)) * p.qs + (long)head * kdim;
#pragma unroll
    for (int mp = 0; mp < NM; ++mp)
#pragma unroll
      for (int s = 0; s < KS; ++s) {
        const int d0 = 32 * s + 8 * g;
        qf[x][mp][s] = d0 < p.dim ? ld16(qrow + mp * p.dim + d0) : uint4_t{0u, 0u, 0u, 0u};
      }
    hs[x] = p.scale * (CAP ? 1.f : kLog2e);
    if (p.tevery > 0) hs[x] *= 1.f + p.tcoef * logf((float)((qpos[x] + 1) / p.tevery + 1));
    if constexpr (CAP) hs[x] *= 2.f * kLog2e / p.cap;
  }

  const int* bt = p.bt + (long)b * p.bt_stride;
  const int krow = 8 * (n16 >> 2) + (n16 & 3);
  auto page_of = [&](int key) { return p.bs_shift >= 0 ? key >> p.bs_shift : key / p.BS; };
  // cached keys past the end of what this workgroup sees are never read: places are clamped to the last one, which the mask hides
  auto key_of = [&](int kb, int t) { return min(kb + krow + 4 * t, k1 - 1); };
  auto vkey_of = [&](int kb) { return min(kb + 8 * g, (k1 - 1) & ~7); };
  int pg[3];
  auto pages = [&](int kb) {
    pg[0] = bt[page_of(key_of(kb, 0))];
    pg[1] = bt[page_of(key_of(kb, 1))];
    pg[2] = bt[page_of(vkey_of(kb))];
  };
  const unsigned lds0 = (unsigned)reinterpret_cast<uintptr_t>((lds_void_ptr)lds);
  auto issue = [&](int kb, int buf) {
    const bf16_t* kr[2];
#pragma unroll
    for (int t = 0; t < 2; ++t) {
      const int key = key_of(kb, t);
      kr[t] = p.kc + (((long)pg[t] * p.G + kvh) * p.BS + (key - page_of(key) * p.BS)) * kdim;
    }
    const int vk = vkey_of(kb);
    const bf16_t* vr = p.vc + ((long)pg[2] * p.G + kvh) * p.vdim * p.BS + (vk - page_of(vk) * p.BS);
#pragma unroll
    for (int i = 0; i < (FR + 3) / 4; ++i) {
      const int f = 4 * i + w;
      if (FR % 4 != 0 && f >= FR) break;
      const unsigned off = lds0 + (unsigned)(buf * FR + f) * 1024u;
      if (f < NK) {
        const int mp = f / (2 * KS), t = f / KS % 2, s = f % KS;
        dma16(off, (t ? kr[1] : kr[0]) + mp * p.dim + min(32 * s + 8 * g, p.dim - 8));   // (columns past dim meet zero queries)
      } else {
        dma16(off, vr + (long)min((f - NK) * 16 + n16, p.vdim - 1) * p.BS);              // (values past vdim are not stored)
      }
    }
  };

  floatx4 o[CG][NM][VT];
  float m[CG][NM], l[CG][NM];
#pragma unroll
  for (int x = 0; x < CG; ++x)
#pragma unroll
    for (int mp = 0; mp < NM; ++mp) {
      m[x][mp] = kNegBig;
      l[x][mp] = 0.f;
#pragma unroll
      for (int vt = 0; vt < VT; ++vt) o[x][mp][vt] = floatx4{0.f, 0.f, 0.f, 0.f};
    }

  pages(0);
  issue(0, 0);
  if (ntile > 1) pages(32);
  for (int tt = 0; tt < ntile; ++tt) {
    const int kb = 32 * tt, buf = tt & 1;
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");   // this wave's part of tile tt has arrived
    __syncthreads();                                   // all of it has, and tile tt - 1 has been consumed
    if (tt + 1 < ntile) {
      issue(kb + 32, buf ^ 1);
      if (tt + 2 < ntile) pages(kb + 64);
    }
    if (kb >= wend) continue;
    const bf16_t* fr = lds + (long)buf * FR * 512 + lane * 8;
    floatx4 c[CG][NM][2];
#pragma unroll
    for (int mp = 0; mp < NM; ++mp)
#pragma unroll
      for (int t = 0; t < 2; ++t) {
#pragma unroll
        for (int x = 0; x < CG; ++x) c[x][mp][t] = floatx4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int s = 0; s < KS; ++s) {
          const uint4_t kf = ld16(fr + ((mp * 2 + t) * KS + s) * 512);
#pragma unroll
          for (int x = 0; x < CG; ++x) c[x][mp][t] = mma_qk<bf16_t>(kf, qf[x][mp][s], c[x][mp][t]);
        }
      }
    const bool edge = kb + 31 > past + qw || kb + 32 > ctx;   // (wave-uniform) some column does not see all 32 keys
    short8 pb[CG][NM];
#pragma unroll
    for (int x = 0; x < CG; ++x)
#pragma unroll
      for (int mp = 0; mp < NM; ++mp) {
        float v[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          v[e] = c[x][mp][e >> 2][e & 3] * hs[x];
          if constexpr (CAP) v[e] = p.cap * kLog2e * (1.f - 2.f * __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(v[e])));
        }
        if (edge) {
          const int last = min(qpos[x], ctx - 1) - kb - 8 * g;
#pragma unroll
          for (int e = 0; e < 8; ++e) v[e] = e <= last ? v[e] : kNegBig;
        }
        float mx = fmaxf(fmaxf(fmaxf(v[0], v[1]), fmaxf(v[2], v[3])), fmaxf(fmaxf(v[4], v[5]), fmaxf(v[6], v[7])));
        mx = max_groups(mx);
        const bool grow = mx > m[x][mp] + kDefer;
        if (__any(grow)) {
          const float mn = grow ? mx : m[x][mp], alpha = __builtin_amdgcn_exp2f(m[x][mp] - mn);
          m[x][mp] = mn;
          l[x][mp] *= alpha;
#pragma unroll
          for (int vt = 0; vt < VT; ++vt)
#pragma unroll
            for (int j = 0; j < 4; ++j) o[x][mp][vt][j] *= alpha;
        }
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          v[e] = __builtin_amdgcn_exp2f(v[e] - m[x][mp]);
          l[x][mp] += v[e];
        }
        uint4_t pk;
#pragma unroll
        for (int e = 0; e < 4; ++e) pk[e] = pack_bf2(v[2 * e], v[2 * e + 1]);
        pb[x][mp] = __builtin_bit_cast(short8, pk);
      }
#pragma unroll
    for (int vt = 0; vt < VT; ++vt) {
      const short8 vf = __builtin_bit_cast(short8, ld16(fr + (NK + vt) * 512));
#pragma unroll
      for (int x = 0; x < CG; ++x)
#pragma unroll
        for (int mp = 0; mp < NM; ++mp) o[x][mp][vt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pb[x][mp], o[x][mp][vt], 0, 0, 0);
    }
  }

#pragma unroll
  for (int x = 0; x < CG; ++x) {
    float f[NM];
#pragma unroll
    for (int mp = 0; mp < NM; ++mp) {
      float t = l[x][mp];
      t += __shfl_xor(t, 16, 64);
      t += __shfl_xor(t, 32, 64);
      f[mp] = t > 0.f ? 1.f / t : 0.f;
    }
    float fo = p.oscale;
    if constexpr (NM == 1) {
      fo *= f[0];
    } else {
      f[1] *= p.lam[0];
      float ss = 0.f;
#pragma unroll
      for (int vt = 0; vt < VT; ++vt)
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const float r = vt * 16 + 4 * g + j < p.vdim ? o[x][0][vt][j] * f[0] - o[x][NM - 1][vt][j] * f[NM - 1] : 0.f;
          o[x][0][vt][j] = r;
          ss += r * r;
        }
      ss += __shfl_xor(ss, 16, 64);
      ss += __shfl_xor(ss, 32, 64);
      fo /= sqrtf(ss * p.inv_nv + p.eps);
    }
    const int qi = qw + 16 * x + n16;
    if (qi >= qlen) continue;
    const bf16_t* gr = p.gate + (long)(qbeg + qi) * p.gs + p.gcol + (long)head * p.vdim;
    bf16_t* orow = out + (long)(qbeg + qi) * os + (long)head * p.vdim;
#pragma unroll
    for (int vt = 0; vt < VT; ++vt) {
      const int vd = vt * 16 + 4 * g;
      if (vd < p.vdim) {   // (vdim is a multiple of 8)
        const short4_t gv = *reinterpret_cast<const short4_t*>(gr + vd);
        short4_t r;
#pragma unroll
        for (int j = 0; j < 4; ++j)
          r[j] = (short)f2bf(o[x][0][vt][j] * fo * __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(-kLog2e * bf2f((bf16_t)gv[j]))));
        *reinterpret_cast<short4_t*>(orow + vd) = r;
      }
    }
  }
}

template <int KP, int VP, int NM, bool CAP>
int launch(const TileParams& p, const int* cu_q, const int* ctx, const int* ts, const int* tq, int ntiles, bf16_t* out, long os, hipStream_t st) {
  constexpr int lds = 2 * (NM * 2 * (KP / 32) + VP / 16) * 1024;
  LK_SET_MAX_LDS((tile_attention_kernel<KP, VP, NM, CAP>), lds);
  tile_attention_kernel<KP, VP, NM, CAP><<<dim3(p.H / p.wh, ntiles), 256, lds, st>>>(p, cu_q, ctx, ts, tq, out, os);
  LK_CHECK_LAUNCH();
  return 0;
}

#define LK_TILE_V(KP, NM, CAP, ...)                        \
  (p.vdim <= 64    ? launch<KP, 64, NM, CAP>(__VA_ARGS__)  \
   : p.vdim <= 128 ? launch<KP, 128, NM, CAP>(__VA_ARGS__) \
                   : launch<KP, 256, NM, CAP>(__VA_ARGS__))
#define LK_TILE(NM, CAP, ...)                              \
  (p.dim <= 32    ? LK_TILE_V(32, NM, CAP, __VA_ARGS__)    \
   : p.dim <= 64  ? LK_TILE_V(64, NM, CAP, __VA_ARGS__)    \
   : p.dim <= 128 ? LK_TILE_V(128, NM, CAP, __VA_ARGS__)   \
                  : LK_TILE_V(256, NM, CAP, __VA_ARGS__))

}  // namespace

// maps 1: softmax attention (cap > 0: capped scores; lam, eps, norm_vdim unused), 2: differential.  The tile list holds entries of
// 32 * 4 / wh queries, wh = the largest of 4, 2, 1 that divides H / G.
int lk_tile_attention_prefill(const void* q, long qs, const void* kc, const void* vc, const int* bt, int bt_stride, const int* cu_q,
                              const int* ctx_lens, const int* tile_seq, const int* tile_q0, int ntiles, int maps, int H, int G, int dim,
                              int vdim, int BS, float scale, float cap, float tcoef, int tevery, const float* lam, float eps, int norm_vdim,
                              float oscale, const void* gate, long gs, int gcol, void* out, long os, hipStream_t st) {
  if (ntiles <= 0) return 0;
  const auto al = [](const void* x, int b) { return reinterpret_cast<uintptr_t>(x) % b == 0; };
  if (maps < 1 || maps > 2 || H < 1 || G < 1 || H % G || dim < 8 || vdim < 8 || dim % 8 || vdim % 8 || dim > 256 || vdim > 256 || BS < 16 ||
      BS % 16 || ntiles > 65535 || tevery < 0 || cap < 0.f || (maps == 2 && (!lam || cap > 0.f)) || norm_vdim < 1 || !gate || qs % 8 ||
      !al(q, 16) || !al(kc, 16) || !al(vc, 16) || !al(gate, 8) || gs % 4 || gcol % 4 || !al(out, 8) || os % 4)
    return -1;
  TileParams p;
  p.q = (const bf16_t*)q; p.qs = qs; p.kc = (const bf16_t*)kc; p.vc = (const bf16_t*)vc; p.bt = bt; p.bt_stride = bt_stride;
  p.H = H; p.G = G; p.dim = dim; p.vdim = vdim; p.BS = BS;
  p.bs_shift = (BS & (BS - 1)) == 0 ? __builtin_ctz(BS) : -1;
  const int rep = H / G;
  p.wh = rep % 4 == 0 ? 4 : rep % 2 == 0 ? 2 : 1;
  p.scale = scale; p.cap = cap; p.tcoef = tcoef; p.tevery = tevery; p.lam = lam; p.eps = eps; p.inv_nv = 1.f / (float)norm_vdim;
  p.oscale = oscale; p.gate = (const bf16_t*)gate; p.gs = gs; p.gcol = gcol;
  bf16_t* o = (bf16_t*)out;
  if (maps == 2) return LK_TILE(2, false, p, cu_q, ctx_lens, tile_seq, tile_q0, ntiles, o, os, st);
  return cap > 0.f ? LK_TILE(1, true, p, cu_q, ctx_lens, tile_seq, tile_q0, ntiles, o, os, st)
                   : LK_TILE(1, false, p, cu_q, ctx_lens, tile_seq, tile_q0, ntiles, o, os, st);
}
