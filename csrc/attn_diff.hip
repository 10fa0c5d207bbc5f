// Differential attention over a paged K/V cache, streamed straight from memory: decode rows (bf16 and f32) and f32 prompts (bf16
// prompts run on the staged kernel of attn_tile.hip).
//
//   s_m(i, j) = scale * temp(i) * <q_(i, h, m), k_(j, g, m)>                 m = 1, 2: the two maps of a head, j <= i
//   a_m(i)    = sum_j softmax_j(s_m(i, .)) v_(j, g)                          both maps average the same values
//   o(i)      = (a_1 - lambda a_2),   out = o / sqrt(mean(o^2) + eps) * oscale * sigmoid(gate)     per head, mean over its values
//   temp(i)   = 1 + coef * ln(floor((i + 1) / every) + 1)                    (every = 0: 1)
//
// K cache [blocks, G, BS, 2 dim] (map 1 behind map 2 in a row), V cache key-contiguous [blocks, G, vdim, BS].  A wave holds 16 columns
// (prompts: 16 consecutive queries of a head; decode: the query heads of a kv group) against 32-key steps with the wave layout of
// attn_sink.hip (S^T = K Q^T, O^T += V^T P^T, P^T from the S^T accumulators without a shuffle): a step's values are fetched once
// and feed both maps.  Running-maximum softmax per map; the four waves of a workgroup take every fourth step and are merged through
// LDS in wave order; decode splits the key range over workgroups as well and a second kernel merges the parts and finishes the row.
#include "common.h"
#include "kernels.h"
#include "attn_frag.h"

namespace {

constexpr float kNegBig = -1e30f;

struct DiffParams {
  const void* q;   // rows of [H * 2 dim]
  long qs;
  const void* kc;
  const void* vc;
  const int* bt;
  int bt_stride;
  int H, G, dim, vdim, BS;
  float scale, tcoef;
  int tevery;
  const float* lam;
  float eps, inv_nv, oscale;
  const void* gate;  // rows aligned with q, column gcol + h * vdim + d
  long gs;
  int gcol;
};

LK_DEVICE float temperature(const DiffParams& p, int pos) {
  return p.tevery > 0 ? 1.f + p.tcoef * logf((float)((pos + 1) / p.tevery + 1)) : 1.f;
}

template <bool EXACT>
LK_DEVICE float exp_f(float x) {
  if constexpr (EXACT) return expf(x);
  else return __expf(x);
}

template <typename T, int KP>
using QFrag = uint4_t[2][KP / (4 * El<T>::V)];

template <typename T, int KP>
LK_DEVICE void load_q(const DiffParams& p, const T* qrow, bool cvalid, QFrag<T, KP>& qf) {
  constexpr int EV = El<T>::V, KS = KP / (4 * EV);
  const int g = (threadIdx.x & 63) >> 4;
#pragma unroll
  for (int mp = 0; mp < 2; ++mp)
#pragma unroll
    for (int s = 0; s < KS; ++s) {
      const int d0 = s * 4 * EV + g * EV;
      qf[mp][s] = (cvalid && d0 < p.dim) ? ld16(qrow + mp * p.dim + d0) : uint4_t{0u, 0u, 0u, 0u};
    }
}

// The columns of this wave against the 32-key steps step0, step0 + stride, ... of keys [k0, k1): k0 a multiple of 32, column n = lane % 16
// sits at position qpos.  m, l, o per map: running maximum (equal in the four lane groups of a column), this lane group's share
// of the sum, O^T accumulators.
template <typename T, int KP, int VP>
LK_DEVICE void diff_run(const DiffParams& p, const QFrag<T, KP>& qf, int kvh, const int* bt, int k0, int k1, int step0, int stride, bool cvalid,
                        int qpos, float hs, float (&m)[2], float (&l)[2], floatx4 (&o)[2][VP / 16]) {
  constexpr int EV = El<T>::V, KS = KP / (4 * EV), VT = VP / 16;
  constexpr bool BF = sizeof(T) == 2;
  const int lane = threadIdx.x & 63, n16 = lane & 15, g = lane >> 4;
  const T* kc = reinterpret_cast<const T*>(p.kc);
  const T* vc = reinterpret_cast<const T*>(p.vc);
  const int krow = 8 * (n16 >> 2) + (n16 & 3);
  // A step's page numbers are read two steps ahead and its K rows one step ahead, as soon as the products have consumed the current
  // ones; its V rows before its own products: the loads of a step fly under the arithmetic of the one before.
  int pk[2], pv;   // pages of the K rows / V columns of the next step to be requested
  auto pages = [&](int kb) {
#pragma unroll
    for (int t = 0; t < 2; ++t) pk[t] = bt[min(kb + krow + 4 * t, k1 - 1) / p.BS];
    pv = bt[min(kb + 8 * g, (k1 - 1) & ~7) / p.BS];
  };
  constexpr bool PF = BF && VP <= 128;   // (wider values fill the registers: their K rows are requested map by map when needed)
  uint4_t kf[PF ? 2 : 1][2][KS];
  auto load_k = [&](int kb, int m0, int m1) {
#pragma unroll
    for (int t = 0; t < 2; ++t) {
      const int key = min(kb + krow + 4 * t, k1 - 1);
      const T* kr = kc + (((long)pk[t] * p.G + kvh) * p.BS + key % p.BS) * 2 * p.dim;
#pragma unroll
      for (int mp = m0; mp < m1; ++mp)
#pragma unroll
        for (int s = 0; s < KS; ++s) {
          const int d0 = s * 4 * EV + g * EV;
          kf[PF ? mp : 0][t][s] = d0 < p.dim ? ld16(kr + mp * p.dim + d0) : uint4_t{0u, 0u, 0u, 0u};
        }
    }
  };
  int kb = k0 + 32 * step0;
  if (kb >= k1) return;
  pages(kb);
  if (PF) load_k(kb, 0, 2);
  for (; kb < k1; kb += 32 * stride) {
    const int vk = min(kb + 8 * g, (k1 - 1) & ~7), kn = kb + 32 * stride;
    const T* vrow = vc + ((long)pv * p.G + kvh) * p.vdim * p.BS + vk % p.BS;
    uint4_t vf[BF ? VT : 1];
    if constexpr (BF) {
#pragma unroll
      for (int vt = 0; vt < VT; ++vt) {
        const int vd = vt * 16 + n16;
        vf[vt] = vd < p.vdim ? ld16(vrow + (long)vd * p.BS) : uint4_t{0u, 0u, 0u, 0u};
      }
    }
    if (PF && kn < k1) pages(kn);
    floatx4 c[2][2];
#pragma unroll
    for (int mp = 0; mp < 2; ++mp) {
      if (!PF) load_k(kb, mp, mp + 1);
#pragma unroll
      for (int t = 0; t < 2; ++t) {
        c[mp][t] = floatx4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int s = 0; s < KS; ++s) c[mp][t] = mma_qk<T>(kf[PF ? mp : 0][t][s], qf[mp][s], c[mp][t]);
      }
    }
    if (kn < k1) {
      if (PF) load_k(kn, 0, 2);
      else pages(kn);
    }
    short8 pbits[2];
    float pw[2][2][4];
#pragma unroll
    for (int mp = 0; mp < 2; ++mp) {
      float mx = kNegBig;
#pragma unroll
      for (int t = 0; t < 2; ++t)
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const int key = kb + 8 * g + 4 * t + j;
          const float s = c[mp][t][j] * hs;
          pw[mp][t][j] = cvalid && key <= qpos && key < k1 ? s : kNegBig;
          mx = fmaxf(mx, pw[mp][t][j]);
        }
      mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
      mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
      const float mn = fmaxf(m[mp], mx);
      const float alpha = exp_f<!BF>(m[mp] - mn);   // nothing seen yet: exp(0) on zeros
      m[mp] = mn;
      l[mp] *= alpha;
#pragma unroll
      for (int vt = 0; vt < VT; ++vt)
#pragma unroll
        for (int j = 0; j < 4; ++j) o[mp][vt][j] *= alpha;
#pragma unroll
      for (int t = 0; t < 2; ++t)
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const float s = pw[mp][t][j];
          const float e = s > 0.5f * kNegBig ? exp_f<!BF>(s - mn) : 0.f;
          pw[mp][t][j] = e;
          l[mp] += e;
          if constexpr (BF) pbits[mp][4 * t + j] = (short)f2bf(e);
        }
    }
    if constexpr (BF) {
#pragma unroll
      for (int vt = 0; vt < VT; ++vt)
        if (vt * 16 < p.vdim) {
#pragma unroll
          for (int mp = 0; mp < 2; ++mp)
            o[mp][vt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(short8, vf[vt]), pbits[mp], o[mp][vt], 0, 0, 0);
        }
    } else {
#pragma unroll
      for (int vt = 0; vt < VT; ++vt) {
        if (vt * 16 < p.vdim) {
          const int vd = vt * 16 + n16;
#pragma unroll
          for (int t = 0; t < 2; ++t) {
            floatx4 a = {0.f, 0.f, 0.f, 0.f};
            if (vd < p.vdim) a = *reinterpret_cast<const floatx4*>(vrow + (long)vd * p.BS + 4 * t);
#pragma unroll
            for (int j = 0; j < 4; ++j)
#pragma unroll
              for (int mp = 0; mp < 2; ++mp) o[mp][vt] = __builtin_amdgcn_mfma_f32_16x16x4f32(a[j], pw[mp][t][j], o[mp][vt], 0, 0, 0);
          }
        }
      }
    }
  }
}

// Merge of the 4 waves' (m, l, O^T) of one map in wave order through LDS; afterwards wave 0 holds, per column, the maximum, the whole
// sum (all lane groups) and O^T relative to the maximum.
template <bool EXACT, int VT>
LK_DEVICE void merge_waves(float& m, float& l, floatx4 (&o)[VT], float (&red)[3][VT][64][4], float (&ml)[3][64][2]) {
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6;
  l += __shfl_xor(l, 16, 64);
  l += __shfl_xor(l, 32, 64);
  __syncthreads();   // (the other map's values have been read)
  if (w > 0) {
    ml[w - 1][lane][0] = m;
    ml[w - 1][lane][1] = l;
#pragma unroll
    for (int vt = 0; vt < VT; ++vt)
#pragma unroll
      for (int j = 0; j < 4; ++j) red[w - 1][vt][lane][j] = o[vt][j];
  }
  __syncthreads();
  if (w == 0) {
    float M = m;
#pragma unroll
    for (int i = 0; i < 3; ++i) M = fmaxf(M, ml[i][lane][0]);
    const float a0 = exp_f<EXACT>(m - M);
    float a[3];
#pragma unroll
    for (int i = 0; i < 3; ++i) a[i] = exp_f<EXACT>(ml[i][lane][0] - M);
    l = ((l * a0 + ml[0][lane][1] * a[0]) + ml[1][lane][1] * a[1]) + ml[2][lane][1] * a[2];
#pragma unroll
    for (int vt = 0; vt < VT; ++vt)
#pragma unroll
      for (int j = 0; j < 4; ++j)
        o[vt][j] = ((o[vt][j] * a0 + red[0][vt][lane][j] * a[0]) + red[1][vt][lane][j] * a[1]) + red[2][vt][lane][j] * a[2];
    m = M;
  }
}

// one wave: the column's two averages subtracted, normed over the head's values (spread over the four lane groups), gated, stored
template <typename T, int VT>
LK_DEVICE void finish_columns(const DiffParams& p, const float (&l)[2], const floatx4 (&o)[2][VT], long row, int head, bool cvalid, T* orow) {
  const int g = (threadIdx.x & 63) >> 4;
  const float lam = p.lam[0], i1 = l[0] > 0.f ? 1.f / l[0] : 0.f, i2 = l[1] > 0.f ? lam / l[1] : 0.f;
  float ss = 0.f;
  floatx4 r[VT];
#pragma unroll
  for (int vt = 0; vt < VT; ++vt)
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      r[vt][j] = vt * 16 + 4 * g + j < p.vdim ? o[0][vt][j] * i1 - o[1][vt][j] * i2 : 0.f;
      ss += r[vt][j] * r[vt][j];
    }
  ss += __shfl_xor(ss, 16, 64);
  ss += __shfl_xor(ss, 32, 64);
  const float f = p.oscale / sqrtf(ss * p.inv_nv + p.eps);
  if (!cvalid) return;
  const T* gr = reinterpret_cast<const T*>(p.gate) + row * p.gs + p.gcol + (long)head * p.vdim;
#pragma unroll
  for (int vt = 0; vt < VT; ++vt)
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int vd = vt * 16 + 4 * g + j;
      if (vd < p.vdim) El<T>::st(orow + vd, r[vt][j] * f / (1.f + expf(-El<T>::ld(gr + vd))));
    }
}

// ---- prompts: blockIdx.x = head, blockIdx.y walks the tile list (16 queries of one sequence each)
template <typename T, int KP, int VP>
__global__ __launch_bounds__(256) void diff_prefill_kernel(DiffParams p, const int* __restrict__ cu_q, const int* __restrict__ ctx_lens,
                                                           const int* __restrict__ tile_seq, const int* __restrict__ tile_q0,
                                                           T* __restrict__ out, long os) {
  constexpr int VT = VP / 16;
  constexpr bool EXACT = sizeof(T) == 4;
  __shared__ float red[3][VT][64][4];
  __shared__ float ml[3][64][2];
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, n16 = lane & 15;
  const int head = blockIdx.x, b = tile_seq[blockIdx.y], q0 = tile_q0[blockIdx.y];
  const int qbeg = cu_q[b], qlen = cu_q[b + 1] - qbeg, ctx = ctx_lens[b], past = ctx - qlen;
  const int qi = q0 + n16, qpos = past + qi;
  const bool cvalid = qi < qlen;
  const T* qrow = reinterpret_cast<const T*>(p.q) + (long)(qbeg + min(qi, qlen - 1)) * p.qs + (long)head * 2 * p.dim;
  QFrag<T, KP> qf;
  load_q<T, KP>(p, qrow, cvalid, qf);
  floatx4 o[2][VT];
  float m[2] = {kNegBig, kNegBig}, l[2] = {0.f, 0.f};
#pragma unroll
  for (int mp = 0; mp < 2; ++mp)
#pragma unroll
    for (int vt = 0; vt < VT; ++vt) o[mp][vt] = floatx4{0.f, 0.f, 0.f, 0.f};
  diff_run<T, KP, VP>(p, qf, head / (p.H / p.G), p.bt + (long)b * p.bt_stride, 0, min(ctx, past + q0 + 16), w, 4, cvalid, qpos,
                      p.scale * temperature(p, qpos), m, l, o);
#pragma unroll
  for (int mp = 0; mp < 2; ++mp) merge_waves<EXACT, VT>(m[mp], l[mp], o[mp], red, ml);
  if (w == 0) finish_columns<T, VT>(p, l, o, qbeg + qi, head, cvalid, out + (long)(qbeg + qi) * os + (long)head * p.vdim);
}

// ---- decode: workgroup = (sequence, up to 16 heads of one kv group, key split z)
// part: [B, H, Z, 2, vdim + 2] f32 = O^T of a map relative to m, then m, l
template <typename T, int KP, int VP>
__global__ __launch_bounds__(256, sizeof(T) == 2 && VP <= 128 && KP <= 64 ? 2 : 1) void diff_decode_kernel(DiffParams p, const int* __restrict__ ctx_lens, int Z, T* __restrict__ out, long os,
                                                          float* __restrict__ part) {
  constexpr int VT = VP / 16;
  constexpr bool EXACT = sizeof(T) == 4;
  __shared__ float red[3][VT][64][4];
  __shared__ float ml[3][64][2];
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, n16 = lane & 15, g = lane >> 4;
  const int rep = p.H / p.G, ngr = (rep + 15) / 16;
  const int b = blockIdx.x, kvh = blockIdx.y / ngr, sub = blockIdx.y % ngr, z = blockIdx.z;
  const int ctx = ctx_lens[b], hn = sub * 16 + n16, head = kvh * rep + min(hn, rep - 1);
  const bool cvalid = hn < rep;
  QFrag<T, KP> qf;
  load_q<T, KP>(p, reinterpret_cast<const T*>(p.q) + (long)b * p.qs + (long)head * 2 * p.dim, cvalid, qf);
  floatx4 o[2][VT];
  float m[2] = {kNegBig, kNegBig}, l[2] = {0.f, 0.f};
#pragma unroll
  for (int mp = 0; mp < 2; ++mp)
#pragma unroll
    for (int vt = 0; vt < VT; ++vt) o[mp][vt] = floatx4{0.f, 0.f, 0.f, 0.f};
  const int nsteps = (ctx + 31) / 32, spz = (nsteps + Z - 1) / Z, s0 = z * spz, s1 = min(nsteps, s0 + spz);
  if (s0 < s1)
    diff_run<T, KP, VP>(p, qf, kvh, p.bt + (long)b * p.bt_stride, 32 * s0, min(ctx, 32 * s1), w, 4, cvalid, ctx - 1,
                        p.scale * temperature(p, ctx - 1), m, l, o);
#pragma unroll
  for (int mp = 0; mp < 2; ++mp) merge_waves<EXACT, VT>(m[mp], l[mp], o[mp], red, ml);
  if (w != 0) return;
  if (Z == 1) {
    finish_columns<T, VT>(p, l, o, b, head, cvalid, out + (long)b * os + (long)head * p.vdim);
  } else if (cvalid) {
#pragma unroll
    for (int mp = 0; mp < 2; ++mp) {
      float* pp = part + ((((long)b * p.H + head) * Z + z) * 2 + mp) * (p.vdim + 2);
#pragma unroll
      for (int vt = 0; vt < VT; ++vt)
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const int vd = vt * 16 + 4 * g + j;
          if (vd < p.vdim) pp[vd] = o[mp][vt][j];
        }
      if (g == 0) {
        pp[p.vdim] = m[mp];
        pp[p.vdim + 1] = l[mp];
      }
    }
  }
}

// one wave per (sequence, head): merges the key splits of both maps and finishes the row (lane d owns the values d, d + 64, ..)
template <typename T>
__global__ __launch_bounds__(64) void diff_reduce_kernel(DiffParams p, const float* __restrict__ part, int Z, T* __restrict__ out, long os) {
  constexpr bool EXACT = sizeof(T) == 4;
  const int b = blockIdx.x, head = blockIdx.y, lane = threadIdx.x, st = p.vdim + 2;
  const float* pp = part + ((long)b * p.H + head) * Z * 2 * st;
  float a[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int mp = 0; mp < 2; ++mp) {
    float M = kNegBig, den = 0.f, s[4] = {0.f, 0.f, 0.f, 0.f};
    for (int z = 0; z < Z; ++z) M = fmaxf(M, pp[(2 * z + mp) * st + p.vdim]);
    for (int z = 0; z < Z; ++z) {
      const float* pz = pp + (2 * z + mp) * st;
      const float f = exp_f<EXACT>(pz[p.vdim] - M);
      den += pz[p.vdim + 1] * f;
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (lane + 64 * i < p.vdim) s[i] += pz[lane + 64 * i] * f;
    }
    const float f = den > 0.f ? (mp ? -p.lam[0] : 1.f) / den : 0.f;
#pragma unroll
    for (int i = 0; i < 4; ++i) a[i] += s[i] * f;
  }
  const float f = p.oscale / sqrtf(wave_sum((a[0] * a[0] + a[1] * a[1]) + (a[2] * a[2] + a[3] * a[3])) * p.inv_nv + p.eps);
  const T* gr = reinterpret_cast<const T*>(p.gate) + (long)b * p.gs + p.gcol + (long)head * p.vdim;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int vd = lane + 64 * i;
    if (vd < p.vdim) El<T>::st(out + (long)b * os + (long)head * p.vdim + vd, a[i] * f / (1.f + expf(-El<T>::ld(gr + vd))));
  }
}

bool shape_ok(const DiffParams& p, int esz) {
  const int ev = 16 / esz;
  return p.H > 0 && p.G > 0 && p.H % p.G == 0 && p.dim > 0 && p.vdim > 0 && p.dim % ev == 0 && p.vdim % ev == 0 && p.dim <= 256 &&
         p.vdim <= 256 && p.BS > 0 && p.BS % 16 == 0 && p.tevery >= 0 && p.lam != nullptr && p.gate != nullptr;
}

template <typename T, int KP, int VP>
int launch_decode(const DiffParams& p, const int* ctx, int B, int Z, void* out, long os, float* part, hipStream_t st) {
  const int rep = p.H / p.G;
  diff_decode_kernel<T, KP, VP><<<dim3(B, p.G * ((rep + 15) / 16), Z), 256, 0, st>>>(p, ctx, Z, reinterpret_cast<T*>(out), os, part);
  LK_CHECK_LAUNCH();
  if (Z > 1) {
    diff_reduce_kernel<T><<<dim3(B, p.H), 64, 0, st>>>(p, part, Z, reinterpret_cast<T*>(out), os);
    LK_CHECK_LAUNCH();
  }
  return 0;
}

template <typename T, int KP, int VP>
int launch_prefill(const DiffParams& p, const int* cu_q, const int* ctx, const int* ts, const int* tq, int ntiles, void* out, long os,
                   hipStream_t st) {
  if (ntiles > 65535) return -2;
  diff_prefill_kernel<T, KP, VP><<<dim3(p.H, ntiles), 256, 0, st>>>(p, cu_q, ctx, ts, tq, reinterpret_cast<T*>(out), os);
  LK_CHECK_LAUNCH();
  return 0;
}

#define LK_DIFF_V(FN, T, KP, ...)                        \
  (p.vdim <= 64    ? FN<T, KP, 64>(__VA_ARGS__)          \
   : p.vdim <= 128 ? FN<T, KP, 128>(__VA_ARGS__)         \
                   : FN<T, KP, 256>(__VA_ARGS__))
#define LK_DIFF(FN, T, ...)                                     \
  (p.dim <= 32    ? LK_DIFF_V(FN, T, 32, __VA_ARGS__)           \
   : p.dim <= 64  ? LK_DIFF_V(FN, T, 64, __VA_ARGS__)           \
   : p.dim <= 128 ? LK_DIFF_V(FN, T, 128, __VA_ARGS__)          \
                  : LK_DIFF_V(FN, T, 256, __VA_ARGS__))

DiffParams make_params(const void* q, long qs, const void* kc, const void* vc, const int* bt, int bt_stride, int H, int G, int dim, int vdim,
                       int BS, float scale, float tcoef, int tevery, const float* lam, float eps, int norm_vdim, float oscale,
                       const void* gate, long gs, int gcol) {
  DiffParams p;
  p.q = q; p.qs = qs; p.kc = kc; p.vc = vc; p.bt = bt; p.bt_stride = bt_stride; p.H = H; p.G = G; p.dim = dim; p.vdim = vdim; p.BS = BS;
  p.scale = scale; p.tcoef = tcoef; p.tevery = tevery; p.lam = lam; p.eps = eps; p.inv_nv = 1.f / (float)norm_vdim; p.oscale = oscale;
  p.gate = gate; p.gs = gs; p.gcol = gcol;
  return p;
}

}  // namespace

// f32 rows (bf16 prompts: lk_tile_attention_prefill)
int lk_diff_attention_prefill(const void* q, long qs, const void* kc, const void* vc, const int* bt, int bt_stride, const int* cu_q,
                              const int* ctx_lens, const int* tile_seq, const int* tile_q0, int ntiles, int H, int G, int dim, int vdim,
                              int BS, float scale, float tcoef, int tevery, const float* lam, float eps, int norm_vdim, float oscale,
                              const void* gate, long gs, int gcol, void* out, long os, int esz, hipStream_t st) {
  if (ntiles <= 0) return 0;
  if (esz != 4 || norm_vdim < 1) return -1;
  const DiffParams p = make_params(q, qs, kc, vc, bt, bt_stride, H, G, dim, vdim, BS, scale, tcoef, tevery, lam, eps, norm_vdim, oscale, gate, gs, gcol);
  if (!shape_ok(p, esz)) return -1;
  return LK_DIFF(launch_prefill, float, p, cu_q, ctx_lens, tile_seq, tile_q0, ntiles, out, os, st);
}

int lk_diff_attention_decode(const void* q, long qs, const void* kc, const void* vc, const int* bt, int bt_stride, const int* ctx_lens, int B,
                             int Z, int H, int G, int dim, int vdim, int BS, float scale, float tcoef, int tevery, const float* lam, float eps,
                             int norm_vdim, float oscale, const void* gate, long gs, int gcol, void* out, long os, float* part, int esz,
                             hipStream_t st) {
  if (B <= 0) return 0;
  if (norm_vdim < 1) return -1;
  const DiffParams p = make_params(q, qs, kc, vc, bt, bt_stride, H, G, dim, vdim, BS, scale, tcoef, tevery, lam, eps, norm_vdim, oscale, gate, gs, gcol);
  if (!shape_ok(p, esz) || Z < 1 || (Z > 1 && part == nullptr)) return -1;
  return esz == 2 ? LK_DIFF(launch_decode, bf16_t, p, ctx_lens, B, Z, out, os, part, st)
                  : LK_DIFF(launch_decode, float, p, ctx_lens, B, Z, out, os, part, st);
}
