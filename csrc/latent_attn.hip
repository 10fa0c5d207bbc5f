// Softmax attention over a cached latent that all query heads share.  A token's cache row is [latent c (RP columns) | rotated key
// part (RDP columns)], KD = RP + RDP; the queries have been brought to it, so
//
//   s(i, j) = scale * <qa_(i, h), row_j>                 for first(i) <= j <= i      (sliding window; 0: causal)
//   p(i, j) = exp(s(i, j)) / (exp(sink_h) + sum_j' exp(s(i, j')))                    (the sink is optional, not scaled)
//   lat_(i, h) = sum_j p(i, j) c_j                       the average goes through the head's value projection afterwards
//
// One row serves scores and values of every head: a tile of 32 rows is staged in LDS once and multiplied with many (query, head)
// columns.  Wave layout: 16 columns against 32 keys,
//   S^T (keys x columns) = rows . qa^T  on v_mfma_f32_16x16x32_bf16 (rows as 16-byte LDS fragments, queries in registers),
//   O^T (latent x columns) += c^T . P^T with c^T by transposed LDS reads (ds_read_b64_tr_b16) and P^T straight from the S^T
//   accumulators (both sides use the key order 4g + j, 16 + 4g + j).
// LDS rows are unpadded multiples of 128 bytes; the 16-byte pieces of a row are XOR-swizzled inside groups of 8 so that both kinds
// of reads spread over the banks.
//
// Prompt portions: a workgroup owns 128 columns = the heads of a block x consecutive queries of one sequence (32
// columns per wave), tiles double-buffered.  Decode rows: a workgroup (4 waves) owns a sequence and a block of at most 16 heads, each wave walks its own
// tiles (LDS-DMA into a wave-private region), merged through LDS; key splits over workgroups are merged by a second kernel.
// f32 rows (and latents wider than the instances) run on a plain kernel, one workgroup per (row, head).
//
// Masks are taken from absolute positions: a prompt cut anywhere, a decode row and a whole prompt are the same sums.
//
// lk_latent_prep / lk_latent_query_rot prepare the operands (norms, rotation in halves, the cache row) in f32.
#include <type_traits>

#include "common.h"
#include "kernels.h"
#include "attn_frag.h"

namespace {

typedef __attribute__((address_space(3))) void* lds_void_ptr;
typedef const __attribute__((address_space(1))) void* gbl_void_ptr;

constexpr float kNegBig = -1e30f;
constexpr float kLog2e = 1.4426950408889634f;

struct LatParams {
  const void* q;       // [rows, H, KD]
  long qs;             // elements between rows
  const void* cache;   // [blocks, BS, KD]
  const int* bt;
  int bt_stride;
  int BS, H, HC, KD, RP;   // HC: heads per block
  int window;          // 0: causal
  float scale;
  const float* sink;   // [H] or null
  void* out;           // [rows, H, RP]
  long os;
};

LK_DEVICE int first_key(int qpos, int window) { return window > 0 ? max(0, qpos - window + 1) : 0; }

LK_DEVICE int swz(int row) { return (row & 6) | ((row >> 3) & 1); }

// A column's weights are 2^(s - m) with m = its largest score in the first tile it sees, not a running maximum: bf16 and f32 keep
// their relative precision at any scale, so sums and accumulators may grow with later, larger scores and are never rescaled
// (a rescale of accumulators that fill the registers costs a copy of all of them).  Only if a score passes m by more than this
// (base 2), the pass over the keys is repeated with m = the largest score of all.
constexpr float kMaxGrowth = 96.f;

// 32 staged rows (keys kb .. kb + 31) against CG groups of 16 columns: a row fragment read from LDS serves all groups.  m: the
// column's reference (kNegBig: no key seen yet), top: its largest score so far (both base 2, equal in the four lane groups of a
// column), l: this lane group's share of the sum, o: O^T accumulators.  qpos < 0: column without a query.
// LDS reads as assembly with explicit waits: the fragments of a tile stream through a ring of registers several places ahead of the
// MFMAs that use them (left to itself the compiler reads, waits and multiplies one fragment at a time when the accumulators fill
// the registers).  LDS reads return in order, so "at most N outstanding" names the oldest ones.
template <int OFF>
LK_DEVICE void lds_read16(uint4_t& v, unsigned addr) {
  asm volatile("ds_read_b128 %0, %1 offset:%2" : "=v"(v) : "v"(addr), "n"(OFF));
}
template <int OFF>
LK_DEVICE void lds_read_tr(short4_t& v, unsigned addr) {
  asm volatile("ds_read_b64_tr_b16 %0, %1 offset:%2" : "=v"(v) : "v"(addr), "n"(OFF));
}
template <int N, typename V>
LK_DEVICE void lds_wait(V& a, V& b) {
  asm volatile("s_waitcnt lgkmcnt(%2)" : "+v"(a), "+v"(b) : "n"(N));
}
template <int N, int I = 0, typename F>
LK_DEVICE void static_for(F&& f) {
  if constexpr (I < N) {
    f(std::integral_constant<int, I>{});
    static_for<N, I + 1>(f);
  }
}

// maximum over the four lane groups (lanes l, l ^ 16, l ^ 32, l ^ 48), in registers
LK_DEVICE float max_groups(float v) {
  // (the swapped pair is taken apart as integers: a bit cast of a vector's element reads element 0)
  const auto a = __builtin_amdgcn_permlane16_swap(__float_as_uint(v), __float_as_uint(v), false, false);
  const unsigned a0 = a[0], a1 = a[1];
  v = fmaxf(__uint_as_float(a0), __uint_as_float(a1));
  const auto b = __builtin_amdgcn_permlane32_swap(__float_as_uint(v), __float_as_uint(v), false, false);
  const unsigned b0 = b[0], b1 = b[1];
  return fmaxf(__uint_as_float(b0), __uint_as_float(b1));
}

template <int RP, int RDP, int CG, bool THIN>
LK_DEVICE void lat_tile(const bf16_t* tile, const uint4_t (&qf)[CG][(RP + RDP) / 32], int kb, const int (&qpos)[CG], const int (&klo)[CG], float s2,
                        float (&m)[CG], float (&top)[CG], float (&l)[CG], floatx4 (&o)[CG][RP / 16]) {
  constexpr int KD = RP + RDP, NKS = KD / 32, VT = RP / 16;
  constexpr int QA = RP > 256 && CG == 1 && THIN ? 3 : 4, VA = 4;   // fragments requested ahead of their products (QA pairs, VA c^T fragments)
  const int lane = threadIdx.x & 63, n16 = lane & 15, g = lane >> 4;
  const unsigned base = (unsigned)reinterpret_cast<uintptr_t>((lds_void_ptr)tile);
  floatx4 c[CG][2];
#pragma unroll
  for (int x = 0; x < CG; ++x) c[x][0] = c[x][1] = floatx4{0.f, 0.f, 0.f, 0.f};
  const int sw = swz(n16);   // (rows n16 and 16 + n16 have the same swizzle)
  const unsigned k0 = base + n16 * KD * 2 + (g ^ sw) * 16, k1 = base + n16 * KD * 2 + ((4 + g) ^ sw) * 16;
  uint4_t kf[QA][2];
  static_for<QA>([&](auto sc_) {
    constexpr int s = decltype(sc_)::value;
    lds_read16<128 * (s / 2)>(kf[s][0], (s & 1) ? k1 : k0);
    lds_read16<128 * (s / 2) + 16 * KD * 2>(kf[s][1], (s & 1) ? k1 : k0);
  });
  static_for<NKS>([&](auto sc_) {
    constexpr int s = decltype(sc_)::value, ahead = (s + QA < NKS ? QA : NKS - s) - 1;
    lds_wait<2 * ahead>(kf[s % QA][0], kf[s % QA][1]);
#pragma unroll
    for (int t = 0; t < 2; ++t)
#pragma unroll
      for (int x = 0; x < CG; ++x) c[x][t] = mma_qk<bf16_t>(kf[s % QA][t], qf[x][s], c[x][t]);
    if constexpr (s + QA < NKS) {
      lds_read16<128 * ((s + QA) / 2)>(kf[s % QA][0], ((s + QA) & 1) ? k1 : k0);
      lds_read16<128 * ((s + QA) / 2) + 16 * KD * 2>(kf[s % QA][1], ((s + QA) & 1) ? k1 : k0);
    }
  });
  // the first c^T fragments travel under the softmax arithmetic
  const int qq = n16 >> 2, pp = n16 & 3, swv = swz(4 * g + qq);   // rows 4g + qq and 16 + 4g + qq have the same swizzle
  const unsigned vr = base + (4 * g + qq) * KD * 2 + 8 * (pp & 1);
  unsigned va[4];
#pragma unroll
  for (int x = 0; x < 4; ++x) va[x] = vr + ((2 * x + (pp >> 1)) ^ swv) * 16;
  short4_t vlo[VA], vhi[VA];
  static_for<VA>([&](auto vc_) {
    constexpr int vt = decltype(vc_)::value;
    lds_read_tr<128 * (vt / 4)>(vlo[vt], va[vt % 4]);
    lds_read_tr<128 * (vt / 4) + 16 * KD * 2>(vhi[vt], va[vt % 4]);
  });
  short8 pb[CG];
#pragma unroll
  for (int x = 0; x < CG; ++x) {
    float sc[2][4];
    bool ok[2][4];
    float mx = kNegBig;
#pragma unroll
    for (int t = 0; t < 2; ++t)
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int key = kb + 16 * t + 4 * g + j;
        ok[t][j] = key <= qpos[x] && key >= klo[x];
        sc[t][j] = c[x][t][j] * s2;
        if (ok[t][j]) mx = fmaxf(mx, sc[t][j]);
      }
    mx = max_groups(mx);
    if (m[x] == kNegBig) m[x] = mx;
    top[x] = fmaxf(top[x], mx);
#pragma unroll
    for (int t = 0; t < 2; ++t)
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const float p = ok[t][j] ? __builtin_amdgcn_exp2f(sc[t][j] - m[x]) : 0.f;
        l[x] += p;
        pb[x][4 * t + j] = (short)f2bf(p);
      }
  }
  static_for<VT>([&](auto vc_) {
    constexpr int vt = decltype(vc_)::value, ahead = (vt + VA < VT ? VA : VT - vt) - 1;
    lds_wait<2 * ahead>(vlo[vt % VA], vhi[vt % VA]);
    const short8 a = __builtin_shufflevector(vlo[vt % VA], vhi[vt % VA], 0, 1, 2, 3, 4, 5, 6, 7);
#pragma unroll
    for (int x = 0; x < CG; ++x) o[x][vt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, pb[x], o[x][vt], 0, 0, 0);
    if constexpr (vt + VA < VT) {
      lds_read_tr<128 * ((vt + VA) / 4)>(vlo[vt % VA], va[(vt + VA) % 4]);
      lds_read_tr<128 * ((vt + VA) / 4) + 16 * KD * 2>(vhi[vt % VA], va[(vt + VA) % 4]);
    }
  });
}

template <int RP, int RDP>
LK_DEVICE void load_q(const bf16_t* qrow, bool valid, uint4_t (&qf)[(RP + RDP) / 32]) {
  const int g = (threadIdx.x & 63) >> 4;
#pragma unroll
  for (int s = 0; s < (RP + RDP) / 32; ++s) qf[s] = valid ? ld16(qrow + 32 * s + 8 * g) : uint4_t{0u, 0u, 0u, 0u};
}

// the page of the 16-key group kg (a multiple of 16, clamped to the sequence's last group): pages hold a multiple of 16 rows, so
// a group lies in one page
LK_DEVICE int group_page(const int* bt, int BS, int kg, int last) { return bt[min(kg, last) / BS]; }

// 64 pieces of 16 bytes (one per lane, `src`) to 1,024 consecutive bytes of LDS at `dst` (wave-uniform), without registers.  Written as
// assembly: the builtin makes the compiler wait for it before every transposed LDS read, also of the other buffer.  The caller
// waits (vmcnt) before the piece is read.
LK_DEVICE void request_piece(const void* src, void* dst) {
  const unsigned off = __builtin_amdgcn_readfirstlane((unsigned)reinterpret_cast<uintptr_t>((lds_void_ptr)dst));
  asm volatile("s_mov_b32 m0, %0\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %1, off" ::"s"(off), "v"(src) : "memory", "m0");
}

constexpr int kPreCols = 128;
// column groups per wave: two where the accumulators of both fit the registers
template <int RP>
constexpr int pre_groups() { return 2; }
template <int RP>
constexpr int pre_waves() { return kPreCols / (16 * pre_groups<RP>()); }

// grid (query tiles, head blocks): tile x is found by walking the sequences (at most ceil(qlen / NQ) tiles each, a sequence's last
// queries first: they see the most keys)
template <int RP, int RDP>
__global__ __launch_bounds__(pre_waves<RP>() * 64, RP >= 256 ? 1 : 2) void lat_prefill_kernel(LatParams p, const int* __restrict__ cu_q, const int* __restrict__ ctx_lens,
                                                                     int nseq) {
  constexpr int KD = RP + RDP, CPR = KD / 8, VT = RP / 16, NCH = 32 * CPR, NL = (NCH / 64 + pre_waves<RP>() - 1) / pre_waves<RP>(),
                CG = pre_groups<RP>();
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];   // two tiles of 32 rows
  const int tid = threadIdx.x, lane = tid & 63, w = __builtin_amdgcn_readfirstlane(tid >> 6), n16 = lane & 15, g = lane >> 4;
  const int NQ = kPreCols / p.HC;
  int b = -1, q0 = 0;
  {
    const int tile = blockIdx.x;
    int acc = 0;
    for (int i = 0; i < nseq; ++i) {
      const int nt = (cu_q[i + 1] - cu_q[i] + NQ - 1) / NQ;
      if (tile < acc + nt) {
        b = i;
        q0 = (nt - 1 - (tile - acc)) * NQ;
        break;
      }
      acc += nt;
    }
  }
  if (b < 0) return;   // the whole workgroup leaves
  const int qbeg = cu_q[b], qlen = cu_q[b + 1] - qbeg, ctx = ctx_lens[b], past = ctx - qlen;
  uint4_t qf[CG][KD / 32];
  floatx4 o[CG][VT];
  float m[CG], top[CG], l[CG];
  int qpos[CG], klo[CG];
#pragma unroll
  for (int x = 0; x < CG; ++x) {
    const int c = 16 * (CG * w + x) + n16, qi = q0 + c / p.HC, head = blockIdx.y * p.HC + c % p.HC;
    const bool valid = c / p.HC < NQ && qi < qlen && head < p.H;
    qpos[x] = valid ? past + qi : -1;
    klo[x] = first_key(qpos[x], p.window);
    load_q<RP, RDP>(reinterpret_cast<const bf16_t*>(p.q) + (long)(qbeg + min(qi, qlen - 1)) * p.qs + (long)min(head, p.H - 1) * KD, valid, qf[x]);
    m[x] = kNegBig;
  }
  const float s2 = p.scale * kLog2e;
  const int k1 = min(ctx, past + q0 + NQ), k0 = first_key(past + q0, p.window) & ~31, last = (k1 - 1) & ~15;
  const int* bt = p.bt + (long)b * p.bt_stride;
  const bf16_t* cache = reinterpret_cast<const bf16_t*>(p.cache);
  // a tile travels from the cache to LDS without registers (LDS-DMA): 64 pieces of 16 bytes per wave instruction, in the order of
  // their places in LDS; the source piece of a place is the one the swizzle puts there
  const int piece0 = 64 * w + lane;
  constexpr int STEP = 64 * pre_waves<RP>();   // pieces per round of the workgroup's waves
  auto request = [&](int kb, int page0, int page1, int which) {
    const int r0 = __builtin_amdgcn_readfirstlane(page0) * p.BS + min(kb, last) % p.BS,
              r1 = __builtin_amdgcn_readfirstlane(page1) * p.BS + min(kb + 16, last) % p.BS;
    unsigned char* dst = smem + which * 64 * KD;
    int r = piece0 / CPR, pos = piece0 % CPR;   // row and place of this lane's piece, stepped from instruction to instruction
    asm volatile("" : "+v"(r), "+v"(pos));      // (recomputed per tile: the registers are worth more than the few operations)
#pragma unroll
    for (int i = 0; i < NL; ++i) {
      const int blk = pre_waves<RP>() * i + w;   // wave-uniform
      if (NCH / 64 % pre_waves<RP>() == 0 || blk < NCH / 64) {
        const int cc = (pos & ~7) | ((pos & 7) ^ swz(r));
        request_piece(cache + (long)((r < 16 ? r0 : r1) + (r & 15)) * KD + cc * 8, dst + blk * 1024);
      }
      r += STEP / CPR;
      pos += STEP % CPR;
      if (pos >= CPR) {
        pos -= CPR;
        ++r;
      }
    }
  };
  for (int pass = 0; pass < 2; ++pass) {
#pragma unroll
    for (int x = 0; x < CG; ++x) {
      top[x] = kNegBig;
      l[x] = 0.f;
#pragma unroll
      for (int vt = 0; vt < VT; ++vt) o[x][vt] = floatx4{0.f, 0.f, 0.f, 0.f};
    }
    request(k0, group_page(bt, p.BS, k0, last), group_page(bt, p.BS, k0 + 16, last), 0);
    int n0 = group_page(bt, p.BS, k0 + 32, last), n1 = group_page(bt, p.BS, k0 + 48, last);   // the pages of the tile to request next
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();
    int cur = 0;
    for (int kb = k0; kb < k1; kb += 32) {
      if (kb + 32 < k1) {
        request(kb + 32, n0, n1, cur ^ 1);
        n0 = group_page(bt, p.BS, kb + 64, last);   // (raw: used, and waited for, in the next round)
        n1 = group_page(bt, p.BS, kb + 80, last);
      }
      lat_tile<RP, RDP, CG, true>(reinterpret_cast<const bf16_t*>(smem + cur * 64 * KD), qf, kb, qpos, klo, s2, m, top, l, o);
      asm volatile("s_waitcnt vmcnt(0)" ::: "memory");   // the next tile has arrived (this wave's part of it)
      __syncthreads();
      cur ^= 1;
    }
    int again = 0;
#pragma unroll
    for (int x = 0; x < CG; ++x) {
      again |= top[x] > m[x] + kMaxGrowth;
      m[x] = pass == 0 && top[x] > m[x] + kMaxGrowth ? top[x] : m[x];
    }
    if (!__syncthreads_or(again)) break;
  }
#pragma unroll
  for (int x = 0; x < CG; ++x) {
    l[x] += __shfl_xor(l[x], 16, 64);
    l[x] += __shfl_xor(l[x], 32, 64);
    const int c = 16 * (CG * w + x) + n16, qi = q0 + c / p.HC, head = blockIdx.y * p.HC + c % p.HC;
    if (qpos[x] >= 0) {
      if (p.sink) l[x] += __builtin_amdgcn_exp2f(p.sink[head] * kLog2e - m[x]);   // one more term without a value
      const float f = l[x] > 0.f ? 1.f / l[x] : 0.f;
      bf16_t* orow = reinterpret_cast<bf16_t*>(p.out) + (long)(qbeg + qi) * p.os + (long)head * RP + 4 * g;
#pragma unroll
      for (int vt = 0; vt < VT; ++vt) {
        short4_t v;
#pragma unroll
        for (int j = 0; j < 4; ++j) v[j] = (short)f2bf(o[x][vt][j] * f);
        *reinterpret_cast<short4_t*>(orow + 16 * vt) = v;
      }
    }
  }
}

// grid (sequences, head blocks, key splits).  part: [B, H, Z, RP + 2] f32 = O^T relative to m (base 2), then m, l
template <int RP, int RDP>
__global__ __launch_bounds__(256) void lat_decode_kernel(LatParams p, const int* __restrict__ ctx_lens, int Z, float* __restrict__ part) {
  constexpr int KD = RP + RDP, CPR = KD / 8, VT = RP / 16, NCH = 32 * CPR;
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];   // 4 wave-private regions of 32 rows
  const int tid = threadIdx.x, lane = tid & 63, w = tid >> 6, n16 = lane & 15, g = lane >> 4;
  const int b = blockIdx.x, z = blockIdx.z, ctx = ctx_lens[b];
  const int head = blockIdx.y * p.HC + n16;
  const bool valid = n16 < p.HC && head < p.H && ctx > 0;
  unsigned char* region = smem + w * 64 * KD;
  const int qpos[1] = {valid ? ctx - 1 : -1}, klo[1] = {first_key(ctx - 1, p.window)}, k0 = klo[0];
  const bf16_t* qrow = reinterpret_cast<const bf16_t*>(p.q) + (long)b * p.qs + (long)min(head, p.H - 1) * KD;
  uint4_t qf[1][KD / 32];
  load_q<RP, RDP>(qrow, valid, qf[0]);
  floatx4 o[1][VT];
  float m[1] = {kNegBig}, top[1], l[1];
  const float s2 = p.scale * kLog2e;
  const int nsteps = ctx > 0 ? (ctx - k0 + 31) / 32 : 0, spz = (nsteps + Z - 1) / Z, e1 = min(nsteps, (z + 1) * spz);
  const int* bt = p.bt + (long)b * p.bt_stride;
  const bf16_t* cache = reinterpret_cast<const bf16_t*>(p.cache);
  for (int pass = 0; pass < 2; ++pass) {
    top[0] = kNegBig;
    l[0] = 0.f;
#pragma unroll
    for (int vt = 0; vt < VT; ++vt) o[0][vt] = floatx4{0.f, 0.f, 0.f, 0.f};
    for (int step = z * spz + w; step < e1; step += 4) {
      const int kb = k0 + 32 * step;
      // tiles start at the first visible key (a window of 32 n keys is n tiles): lane x looks up the cache row of key kb + x % 32
      const int key = min(kb + (lane & 31), ctx - 1), mine = bt[key / p.BS] * p.BS + key % p.BS;
      asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");   // the previous tile's LDS reads are done
  #pragma unroll
      for (int i = 0; i < NCH / 64; ++i) {
        // LDS piece x = 64 i + lane of the region is position x % CPR of row x / CPR: it holds the source piece swizzled back
        const int x = 64 * i + lane, r = x / CPR, pos = x % CPR, cc = (pos & ~7) | ((pos & 7) ^ swz(r));
        __builtin_amdgcn_global_load_lds((gbl_void_ptr)(cache + (long)__shfl(mine, r, 64) * KD + cc * 8), (lds_void_ptr)(region + i * 1024), 16, 0, 0);
      }
      asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
      lat_tile<RP, RDP, 1, false>(reinterpret_cast<const bf16_t*>(region), qf, kb, qpos, klo, s2, m, top, l, o);
    }
    if (!__any(top[0] > m[0] + kMaxGrowth)) break;
    m[0] = top[0] > m[0] + kMaxGrowth ? top[0] : m[0];
  }
  // ---- merge the 4 waves: (m, l) behind every region's O block, then O relative to the common maximum
  l[0] += __shfl_xor(l[0], 16, 64);
  l[0] += __shfl_xor(l[0], 32, 64);
  asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
  float* ml = reinterpret_cast<float*>(region + 64 * RP);   // RP * 16 f32 of O come first; KD > RP leaves room behind them
  if (g == 0) {
    ml[n16] = m[0];
    ml[16 + n16] = l[0];
  }
  __syncthreads();
  // (the sink is one more term without a value, counted by the first split)
  const float sk = p.sink && z == 0 ? p.sink[min(head, p.H - 1)] * kLog2e : kNegBig;
  float M = sk, L = 0.f;
#pragma unroll
  for (int i = 0; i < 4; ++i) M = fmaxf(M, reinterpret_cast<const float*>(smem + i * 64 * KD + 64 * RP)[n16]);
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const float* q = reinterpret_cast<const float*>(smem + i * 64 * KD + 64 * RP);
    L += q[16 + n16] * __builtin_amdgcn_exp2f(q[n16] - M);
  }
  if (p.sink && z == 0) L += __builtin_amdgcn_exp2f(sk - M);
  const float f = __builtin_amdgcn_exp2f(m[0] - M);
  floatx4* ob = reinterpret_cast<floatx4*>(region);
#pragma unroll
  for (int vt = 0; vt < VT; ++vt) ob[vt * 64 + lane] = floatx4{o[0][vt][0] * f, o[0][vt][1] * f, o[0][vt][2] * f, o[0][vt][3] * f};
  __syncthreads();
  const float inv = L > 0.f ? 1.f / L : 0.f;
#pragma unroll
  for (int i = 0; i < VT / 4; ++i) {
    const int vt = 4 * i + w;
    floatx4 s = reinterpret_cast<const floatx4*>(smem)[vt * 64 + lane];
#pragma unroll
    for (int x = 1; x < 4; ++x) {
      const floatx4 t = reinterpret_cast<const floatx4*>(smem + x * 64 * KD)[vt * 64 + lane];
#pragma unroll
      for (int j = 0; j < 4; ++j) s[j] += t[j];
    }
    if (n16 < p.HC && head < p.H) {
      if (Z == 1) {
        short4_t v;
#pragma unroll
        for (int j = 0; j < 4; ++j) v[j] = (short)f2bf(s[j] * inv);
        *reinterpret_cast<short4_t*>(reinterpret_cast<bf16_t*>(p.out) + (long)b * p.os + (long)head * RP + 16 * vt + 4 * g) = v;
      } else {
        float* pp = part + (((long)b * p.H + head) * Z + z) * (RP + 2) + 16 * vt + 4 * g;
#pragma unroll
        for (int j = 0; j < 4; ++j) pp[j] = s[j];
      }
    }
  }
  if (Z > 1 && w == 0 && g == 0 && n16 < p.HC && head < p.H) {
    float* pp = part + (((long)b * p.H + head) * Z + z) * (RP + 2) + RP;
    pp[0] = M;
    pp[1] = L;
  }
}

__global__ __launch_bounds__(256) void lat_reduce_kernel(LatParams p, const float* __restrict__ part, int Z) {
  const int b = blockIdx.x, head = blockIdx.y, RP = p.RP;
  const float* pp = part + ((long)b * p.H + head) * Z * (RP + 2);
  float M = kNegBig, L = 0.f;
  for (int z = 0; z < Z; ++z) M = fmaxf(M, pp[(long)z * (RP + 2) + RP]);
  for (int z = 0; z < Z; ++z) L += pp[(long)z * (RP + 2) + RP + 1] * __builtin_amdgcn_exp2f(pp[(long)z * (RP + 2) + RP] - M);
  const float inv = L > 0.f ? 1.f / L : 0.f;
  for (int d = threadIdx.x; d < RP; d += 256) {
    float s = 0.f;
    for (int z = 0; z < Z; ++z) s += pp[(long)z * (RP + 2) + d] * __builtin_amdgcn_exp2f(pp[(long)z * (RP + 2) + RP] - M);
    reinterpret_cast<bf16_t*>(p.out)[(long)b * p.os + (long)head * RP + d] = f2bf(s * inv);
  }
}

// ---- plain form: one workgroup per (row, head), keys in rounds of 256 (one per thread for the scores, all threads over the
// latent's columns for the average).  cu_q null: decode rows.
constexpr int kPlainDims = 8;   // latent columns per thread: RP <= 2048

template <typename T>
__global__ __launch_bounds__(256) void lat_plain_kernel(LatParams p, const int* __restrict__ cu_q, const int* __restrict__ ctx_lens, int nseq) {
  constexpr bool EXACT = sizeof(T) == 4;
  extern __shared__ __attribute__((aligned(16))) unsigned char smem[];
  float* q = reinterpret_cast<float*>(smem);          // [KD]
  float* pw = q + p.KD;                                // [256]
  long* rows = reinterpret_cast<long*>(pw + 256);      // [256] element offsets of the cache rows
  __shared__ float red[4];
  const int row = blockIdx.x, head = blockIdx.y, tid = threadIdx.x;
  int b = row, qpos;
  if (cu_q) {
    for (b = 0; b < nseq - 1 && row >= cu_q[b + 1]; ++b) {}
    qpos = ctx_lens[b] - (cu_q[b + 1] - row);
  } else {
    qpos = ctx_lens[b] - 1;
  }
  T* orow = reinterpret_cast<T*>(p.out) + (long)row * p.os + (long)head * p.RP;
  if (qpos < 0) {
    for (int d = tid; d < p.RP; d += 256) El<T>::st(orow + d, 0.f);
    return;
  }
  const T* qrow = reinterpret_cast<const T*>(p.q) + (long)row * p.qs + (long)head * p.KD;
  for (int d = tid; d < p.KD; d += 256) q[d] = El<T>::ld(qrow + d) * p.scale;
  const int* bt = p.bt + (long)b * p.bt_stride;
  const T* cache = reinterpret_cast<const T*>(p.cache);
  float m = p.sink ? p.sink[head] : kNegBig, l = p.sink ? 1.f : 0.f;
  float acc[kPlainDims];
#pragma unroll
  for (int i = 0; i < kPlainDims; ++i) acc[i] = 0.f;
  for (int k0 = first_key(qpos, p.window); k0 <= qpos; k0 += 256) {
    const int n = min(256, qpos + 1 - k0);
    __syncthreads();   // q is there; the previous round's weights have been read
    float s = kNegBig;
    if (tid < n) {
      const int key = k0 + tid;
      const long off = ((long)bt[key / p.BS] * p.BS + key % p.BS) * p.KD;
      rows[tid] = off;
      const T* kr = cache + off;
      float a[4] = {0.f, 0.f, 0.f, 0.f};
      for (int d = 0; d < p.KD; d += 4)
#pragma unroll
        for (int e = 0; e < 4; ++e) a[e] += q[d + e] * El<T>::ld(kr + d + e);
      s = (a[0] + a[1]) + (a[2] + a[3]);
    }
    float mx = wave_max(s);
    if ((tid & 63) == 0) red[tid >> 6] = mx;
    __syncthreads();
    mx = fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3]));
    const float mn = fmaxf(m, mx);
    const float alpha = EXACT ? expf(m - mn) : __expf(m - mn);
    const float w = tid < n ? (EXACT ? expf(s - mn) : __expf(s - mn)) : 0.f;
    pw[tid] = w;
    m = mn;
    l = l * alpha + block_sum<4>(w, red);   // (its barriers also publish pw and rows)
#pragma unroll
    for (int i = 0; i < kPlainDims; ++i) {
      const int d = tid + 256 * i;
      if (d < p.RP) {
        float v = acc[i] * alpha;
        for (int k = 0; k < n; ++k) v += pw[k] * El<T>::ld(cache + rows[k] + d);
        acc[i] = v;
      }
    }
  }
  const float inv = l > 0.f ? 1.f / l : 0.f;
#pragma unroll
  for (int i = 0; i < kPlainDims; ++i) {
    const int d = tid + 256 * i;
    if (d < p.RP) El<T>::st(orow + d, acc[i] * inv);
  }
}

// ---- operands ------------------------------------------------------------------------------------------------------
struct PrepParams {
  const void* u;
  long us;
  int dq, qr;
  const float* wq;
  int dkv, R;
  const float* wkv;    // null: no cache row
  int rd;
  const float* freq;
  const int* positions;
  float eps;
  void* cache;
  const int* slots;
  int RP, KD;
  void* cq;
  long cqs;
};

// One workgroup per token: both root mean squares in one pass over the row, the normed query latent, the cache row.
template <typename T>
__global__ __launch_bounds__(256) void latent_prep_kernel(PrepParams p) {
  __shared__ float red[2][4];
  const long t = blockIdx.x;
  const int tid = threadIdx.x;
  const T* uq = reinterpret_cast<const T*>(p.u) + t * p.us + p.dq;
  const T* ukv = reinterpret_cast<const T*>(p.u) + t * p.us + p.dkv;
  float sq = 0.f, sk = 0.f;
  for (int c = tid; c < p.qr; c += 256) {
    const float v = El<T>::ld(uq + c);
    sq += v * v;
  }
  const int slot = p.wkv ? p.slots[t] : -1;
  if (p.wkv)
    for (int c = tid; c < p.R; c += 256) {
      const float v = El<T>::ld(ukv + c);
      sk += v * v;
    }
  sq = block_sum<4>(sq, red[0]);
  T* cq = reinterpret_cast<T*>(p.cq) + t * p.cqs;
  const float iq = 1.f / sqrtf(sq / (float)p.qr + p.eps);
  for (int c = tid; c < p.qr; c += 256) El<T>::st(cq + c, El<T>::ld(uq + c) * iq * p.wq[c]);
  if (slot < 0) return;   // the same for the whole workgroup
  sk = block_sum<4>(sk, red[1]);
  const float ik = 1.f / sqrtf(sk / (float)p.R + p.eps);
  T* row = reinterpret_cast<T*>(p.cache) + (long)slot * p.KD;   // pages are contiguous: slot = block * BS + offset
  for (int c = tid; c < p.RP; c += 256) El<T>::st(row + c, c < p.R ? El<T>::ld(ukv + c) * ik * p.wkv[c] : 0.f);
  const int half = p.rd / 2;
  const float pos = (float)p.positions[t];
  for (int i = tid; i < half; i += 256) {
    float sn, cs;
    sincosf(pos * p.freq[i], &sn, &cs);
    const float a = El<T>::ld(ukv + p.R + i), b = El<T>::ld(ukv + p.R + half + i);
    El<T>::st(row + p.RP + i, a * cs - b * sn);
    El<T>::st(row + p.RP + half + i, b * cs + a * sn);
  }
  for (int c = p.RP + p.rd + tid; c < p.KD; c += 256) El<T>::st(row + c, 0.f);
}

constexpr int kRotMax = 1024;

// One workgroup per token: cos and sin once per pair, then every head's rotated columns.
template <typename T>
__global__ __launch_bounds__(256) void latent_query_rot_kernel(const T* __restrict__ q, long qs, T* __restrict__ qa, long as, int H, int qdim,
                                                               int dim, int rd, const float* __restrict__ freq,
                                                               const int* __restrict__ positions, int RP, int KD) {
  __shared__ float cs[kRotMax / 2], sn[kRotMax / 2];
  const long t = blockIdx.x;
  const int half = rd / 2, RDP = KD - RP;
  const float pos = (float)positions[t];
  for (int i = threadIdx.x; i < half; i += 256) sincosf(pos * freq[i], &sn[i], &cs[i]);
  __syncthreads();
  for (int x = threadIdx.x; x < H * RDP; x += 256) {
    const int h = x / RDP, d = x % RDP;
    float v = 0.f;
    if (d < rd) {
      const T* s = q + t * qs + (long)h * qdim + dim;
      v = d < half ? El<T>::ld(s + d) * cs[d] - El<T>::ld(s + half + d) * sn[d]
                   : El<T>::ld(s + d) * cs[d - half] + El<T>::ld(s + d - half) * sn[d - half];
    }
    El<T>::st(qa + t * as + (long)h * KD + RP + d, v);
  }
}

bool mfma_shape(int RP, int KD) {
  const int rdp = KD - RP;
  return (RP == 128 || RP == 256 || RP == 512) && (rdp == 64 || rdp == 128);
}

#define LK_LAT_DISPATCH(FN, ...)                                  \
  switch (p.RP * 1000 + p.KD - p.RP) {                            \
    case 128064: return FN<128, 64>(__VA_ARGS__);                 \
    case 128128: return FN<128, 128>(__VA_ARGS__);                \
    case 256064: return FN<256, 64>(__VA_ARGS__);                 \
    case 256128: return FN<256, 128>(__VA_ARGS__);                \
    case 512064: return FN<512, 64>(__VA_ARGS__);                 \
    case 512128: return FN<512, 128>(__VA_ARGS__);                \
    default: return -1;                                           \
  }

template <int RP, int RDP>
int launch_prefill(const LatParams& p, const int* cu_q, const int* ctx, int nseq, long rows, hipStream_t st) {
  constexpr size_t lds = 2 * 64 * (RP + RDP);
  const int NQ = kPreCols / p.HC;
  const long tiles = (rows + NQ - 1) / NQ + nseq;   // every sequence ends with at most one partial tile
  LK_SET_MAX_LDS((lat_prefill_kernel<RP, RDP>), lds);
  lat_prefill_kernel<RP, RDP><<<dim3((unsigned)tiles, (unsigned)((p.H + p.HC - 1) / p.HC)), pre_waves<RP>() * 64, lds, st>>>(p, cu_q, ctx, nseq);
  LK_CHECK_LAUNCH();
  return 0;
}

template <int RP, int RDP>
int launch_decode(const LatParams& p, const int* ctx, int B, int Z, float* part, hipStream_t st) {
  constexpr size_t lds = 4 * 64 * (RP + RDP);
  LK_SET_MAX_LDS((lat_decode_kernel<RP, RDP>), lds);
  lat_decode_kernel<RP, RDP><<<dim3((unsigned)B, (unsigned)((p.H + p.HC - 1) / p.HC), (unsigned)Z), 256, lds, st>>>(p, ctx, Z, part);
  LK_CHECK_LAUNCH();
  if (Z > 1) {
    lat_reduce_kernel<<<dim3((unsigned)B, (unsigned)p.H), 256, 0, st>>>(p, part, Z);
    LK_CHECK_LAUNCH();
  }
  return 0;
}

int run_prefill(const LatParams& p, const int* cu_q, const int* ctx, int nseq, long rows, hipStream_t st) {
  LK_LAT_DISPATCH(launch_prefill, p, cu_q, ctx, nseq, rows, st)
}

int run_decode(const LatParams& p, const int* ctx, int B, int Z, float* part, hipStream_t st) {
  LK_LAT_DISPATCH(launch_decode, p, ctx, B, Z, part, st)
}

template <typename T>
int run_plain(const LatParams& p, const int* cu_q, const int* ctx, int nseq, long rows, hipStream_t st) {
  const size_t lds = sizeof(float) * (p.KD + 256) + sizeof(long) * 256;
  if (p.RP > 256 * kPlainDims || lds > 64 * 1024 || rows > 2147483647L) return -1;
  lat_plain_kernel<T><<<dim3((unsigned)rows, (unsigned)p.H), 256, lds, st>>>(p, cu_q, ctx, nseq);
  LK_CHECK_LAUNCH();
  return 0;
}

bool make_params(LatParams& p, const void* q, long qs, const void* cache, const int* bt, int bt_stride, int BS, int H, int KD, int RP, int window,
                 float scale, const float* sink, void* out, long os, int esz) {
  p.q = q; p.qs = qs; p.cache = cache; p.bt = bt; p.bt_stride = bt_stride; p.BS = BS; p.H = H; p.KD = KD; p.RP = RP; p.window = window;
  p.scale = scale; p.sink = sink; p.out = out; p.os = os;
  const int blocks = (H + 15) / 16;
  p.HC = blocks > 0 ? (H + blocks - 1) / blocks : 1;
  const auto a16 = [](const void* x) { return reinterpret_cast<uintptr_t>(x) % 16 == 0; };
  return H >= 1 && H <= 65535 && BS >= 16 && BS % 16 == 0 && RP >= 16 && KD > RP && KD % 64 == 0 && RP % 64 == 0 && window >= 0 && a16(q) &&
         a16(cache) && a16(out) && qs % (16 / esz) == 0 && os % (16 / esz) == 0;
}

}  // namespace

int lk_latent_attn_prefill(const void* q, long qs, const void* cache, const int* bt, int bt_stride, const int* cu_q, const int* ctx_lens, int nseq,
                           long rows, int BS, int H, int KD, int RP, int window, float scale, const float* sink, void* out, long os, int esz,
                           hipStream_t st) {
  if (rows <= 0 || nseq <= 0) return 0;
  LatParams p;
  if (!make_params(p, q, qs, cache, bt, bt_stride, BS, H, KD, RP, window, scale, sink, out, os, esz)) return -1;
  if (esz == 2 && mfma_shape(RP, KD)) return run_prefill(p, cu_q, ctx_lens, nseq, rows, st);
  return esz == 2 ? run_plain<bf16_t>(p, cu_q, ctx_lens, nseq, rows, st) : run_plain<float>(p, cu_q, ctx_lens, nseq, rows, st);
}

int lk_latent_attn_decode(const void* q, long qs, const void* cache, const int* bt, int bt_stride, const int* ctx_lens, int B, int Z, int BS, int H,
                          int KD, int RP, int window, float scale, const float* sink, void* out, long os, float* part, int esz, hipStream_t st) {
  if (B <= 0) return 0;
  LatParams p;
  if (!make_params(p, q, qs, cache, bt, bt_stride, BS, H, KD, RP, window, scale, sink, out, os, esz)) return -1;
  if (esz == 2 && mfma_shape(RP, KD)) {
    if (Z < 1 || Z > 65535 || (Z > 1 && !part)) return -1;
    return run_decode(p, ctx_lens, B, Z, part, st);
  }
  return esz == 2 ? run_plain<bf16_t>(p, nullptr, ctx_lens, B, B, st) : run_plain<float>(p, nullptr, ctx_lens, B, B, st);
}

int lk_latent_prep(const void* u, long us, int dq, int qr, const float* wq, int dkv, int R, const float* wkv, int rd, const float* freq,
                   const int* positions, float eps, void* cache, const int* slots, int RP, int KD, void* cq, long cqs, long rows, int esz,
                   hipStream_t st) {
  if (rows <= 0) return 0;
  if (qr < 1 || !wq || (wkv && (R < 1 || R > RP || rd < 0 || rd % 2 || RP + rd > KD || !cache || !slots || (rd > 0 && !freq)))) return -1;
  PrepParams p;
  p.u = u; p.us = us; p.dq = dq; p.qr = qr; p.wq = wq; p.dkv = dkv; p.R = R; p.wkv = wkv; p.rd = rd; p.freq = freq; p.positions = positions;
  p.eps = eps; p.cache = cache; p.slots = slots; p.RP = RP; p.KD = KD; p.cq = cq; p.cqs = cqs;
  if (esz == 2) latent_prep_kernel<bf16_t><<<(unsigned)rows, 256, 0, st>>>(p);
  else latent_prep_kernel<float><<<(unsigned)rows, 256, 0, st>>>(p);
  LK_CHECK_LAUNCH();
  return 0;
}

int lk_latent_query_rot(const void* q, long qs, void* qa, long as, int H, int qdim, int dim, int rd, const float* freq, const int* positions, int RP,
                        int KD, long rows, int esz, hipStream_t st) {
  if (rows <= 0) return 0;
  if (H < 1 || rd < 0 || rd % 2 || rd > kRotMax || dim < 0 || dim + rd > qdim || RP + rd > KD || (rd > 0 && !freq)) return -1;
  if (esz == 2)
    latent_query_rot_kernel<bf16_t><<<(unsigned)rows, 256, 0, st>>>((const bf16_t*)q, qs, (bf16_t*)qa, as, H, qdim, dim, rd, freq, positions, RP, KD);
  else
    latent_query_rot_kernel<float><<<(unsigned)rows, 256, 0, st>>>((const float*)q, qs, (float*)qa, as, H, qdim, dim, rd, freq, positions, RP, KD);
  LK_CHECK_LAUNCH();
  return 0;
}
