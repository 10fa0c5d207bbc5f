// Matrix memory with exponential gates: per head and sequence, from log input gates i_t and log forget gates f_t,
//
//   m_t = max(f_t + m_(t-1), i_t)                                   m_0 = 0
//   S_t = exp(f_t + m_(t-1) - m_t) S_(t-1) + exp(i_t - m_t) k_t v_t^T          n_t likewise with k_t alone
//   o_t = S_t^T q_t / (max(|n_t . q_t|, exp(-m_t)) + 1e-6)
//
// q, k, v rows in bf16 or f32; gates, state and everything in between f32.  S [slots, H, dk, dv]; beside it n and m, one copy per
// block of 64 state columns ([slots, H, Z, dk + 4], m behind n), since the workgroups of a head run independently.
//
// A batch is a list of sequences (prompt portions of any length, decode rows of length 1): rows [cu[s], cu[s+1]) belong to
// sequence s, whose state lives in slot slots[s] (< 0: a padding row, its output rows are zeroed) and starts from zero when its
// first row sits at position 0.
#include "common.h"
#include "kernels.h"

namespace {

template <typename T>
LK_DEVICE float ldf(const T* p);
template <>
LK_DEVICE float ldf<bf16_t>(const bf16_t* p) { return bf2f(*p); }
template <>
LK_DEVICE float ldf<float>(const float* p) { return *p; }

constexpr int kColBlock = 64;    // state columns of a workgroup
constexpr int kChunkMin = 8;     // from this many rows of some sequence on: the chunked form
constexpr float kDenEps = 1e-6f;

struct MlstmParams {
  const void* q;
  const void* k;
  const void* v;
  long qs, ks, vs;
  const float* gates;  // rows of 2 H: log input gates, log forget gates
  long gs;
  float q_scale;
  float* S;
  float* nm;
  const int* cu;
  const int* slots;
  const int* positions;
  float* o;
  long os;
  int H, dk, dv, Z;
};

LK_DEVICE void zero_rows(const MlstmParams& a, int row0, int len, int h, int j0, int nthreads) {
  for (int i = threadIdx.x; i < len * kColBlock; i += nthreads) {
    const int c = j0 + i % kColBlock;
    if (c < a.dv) a.o[(long)(row0 + i / kColBlock) * a.os + (long)h * a.dv + c] = 0.f;
  }
}

// ---- token by token (decode rows, very short portions): the state streams through registers once per step.
// grid (sequence, head, column block).  256 threads = 16 groups of 4 adjacent columns x 16 row slices; a thread holds the rows
// rs, rs + 16, ... of its 4 columns (16-byte accesses, VEC).
template <typename T, int NR, bool VEC>
__global__ __launch_bounds__(256) void mlstm_step_kernel(MlstmParams a) {
  __shared__ float sq[NR * 16], sk[NR * 16], red[4][16][5];
  const int s = blockIdx.x, h = blockIdx.y, z = blockIdx.z, j0 = z * kColBlock, tid = threadIdx.x;
  const int row0 = a.cu[s], len = a.cu[s + 1] - row0, slot = a.slots[s];
  if (len <= 0) return;
  if (slot < 0) {
    zero_rows(a, row0, len, h, j0, 256);
    return;
  }
  const int cg = tid & 15, rs = tid >> 4, wv = tid >> 6, lane = tid & 63, c0 = j0 + 4 * cg;
  const bool fresh = a.positions[row0] == 0;
  float* Sg = a.S + ((long)slot * a.H + h) * a.dk * a.dv + c0;
  float* nmg = a.nm + (((long)slot * a.H + h) * a.Z + z) * (a.dk + 4);
  floatx4 S[NR];
  float n[NR];
#pragma unroll
  for (int ii = 0; ii < NR; ++ii) {
    const int i = rs + 16 * ii;
    S[ii] = floatx4{0.f, 0.f, 0.f, 0.f};
    n[ii] = 0.f;
    if (!fresh && i < a.dk) {
      n[ii] = nmg[i];
      if constexpr (VEC) {
        if (c0 < a.dv) S[ii] = *reinterpret_cast<const floatx4*>(Sg + (long)i * a.dv);
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (c0 + e < a.dv) S[ii][e] = Sg[(long)i * a.dv + e];
      }
    }
  }
  float m = fresh ? 0.f : nmg[a.dk];
  const T* qg = reinterpret_cast<const T*>(a.q) + (long)h * a.dk;
  const T* kg = reinterpret_cast<const T*>(a.k) + (long)h * a.dk;
  const T* vg = reinterpret_cast<const T*>(a.v) + (long)h * a.dv;
  for (int t = 0; t < len; ++t) {
    const long row = row0 + t;
    __syncthreads();   // the previous token's operands and sums have been read
    for (int i = tid; i < NR * 16; i += 256) {
      sq[i] = i < a.dk ? ldf<T>(qg + row * a.qs + i) * a.q_scale : 0.f;
      sk[i] = i < a.dk ? ldf<T>(kg + row * a.ks + i) : 0.f;
    }
    float v[4];
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] = c0 + e < a.dv ? ldf<T>(vg + row * a.vs + c0 + e) : 0.f;
    const float ig = a.gates[row * a.gs + h], fg = a.gates[row * a.gs + a.H + h];
    const float mn = fmaxf(fg + m, ig), fa = expf(fg + m - mn), ia = expf(ig - mn);
    m = mn;
    __syncthreads();
    float acc[5] = {0.f, 0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ii = 0; ii < NR; ++ii) {
      const int i = rs + 16 * ii;
      const float kk = ia * sk[i], qq = sq[i];
      n[ii] = fa * n[ii] + kk;
      acc[4] += n[ii] * qq;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        S[ii][e] = fa * S[ii][e] + kk * v[e];
        acc[e] += S[ii][e] * qq;
      }
    }
#pragma unroll
    for (int e = 0; e < 5; ++e) {
      acc[e] += __shfl_xor(acc[e], 16, 64);
      acc[e] += __shfl_xor(acc[e], 32, 64);
    }
    if (lane < 16) {
#pragma unroll
      for (int e = 0; e < 5; ++e) red[wv][lane][e] = acc[e];
    }
    __syncthreads();
    if (tid < 64) {   // thread = (column group, column in it)
      const int g4 = tid >> 2, e = tid & 3;
      const float num = (red[0][g4][e] + red[1][g4][e]) + (red[2][g4][e] + red[3][g4][e]);
      const float nq = (red[0][g4][4] + red[1][g4][4]) + (red[2][g4][4] + red[3][g4][4]);
      const int c = j0 + tid;
      if (c < a.dv) a.o[row * a.os + (long)h * a.dv + c] = num / (fmaxf(fabsf(nq), expf(-m)) + kDenEps);
    }
  }
#pragma unroll
  for (int ii = 0; ii < NR; ++ii) {
    const int i = rs + 16 * ii;
    if (i < a.dk) {
      if constexpr (VEC) {
        if (c0 < a.dv) *reinterpret_cast<floatx4*>(Sg + (long)i * a.dv) = S[ii];
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (c0 + e < a.dv) Sg[(long)i * a.dv + e] = S[ii][e];
      }
      if (cg == 0) nmg[i] = n[ii];
    }
  }
  if (tid == 0) nmg[a.dk] = m;
}

// ---- chunked matrix form (prompt portions): the recurrence unrolled over chunks of 16 tokens, products on true-f32 MFMAs
// (bf16 rows: the q.k products on bf16 MFMAs, exact products either way), the state in the accumulators' layout from
// chunk to chunk.  With F_t = f_1 + .. + f_t inside the chunk, S, n, m the state before it, a_s = i_s - F_s:
//   m_t = F_t + max(m, max_{s<=t} a_s),   c_t = F_t - m_t
//   D_ts = exp(c_t + a_s)  (s <= t),     e_t = exp(c_t + m)
//   num_t = e_t S^T q_t + sum_s D_ts (q_t.k_s) v_s,      nq_t = e_t n.q_t + sum_s D_ts (q_t.k_s)
//   S' = e_L S + sum_s D_Ls k_s v_s^T,   n' = e_L n + sum_s D_Ls k_s,   m' = m_L
// Nothing of a_s, c_t, e_t depends on S: a kernel of one wave per (sequence, head) runs over the gates first and leaves
// (a_t, c_t, c_t + m, m_t) per token, so the chain of the chunk kernel is S alone.
constexpr int kChunk = 16;

template <int N>
LK_DEVICE float row_shr(float old, float v) {   // lane i of a row of 16 gets lane i - N (the first N lanes: old)
  return __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(__builtin_bit_cast(int, old), __builtin_bit_cast(int, v), 0x110 + N, 0xf, 0xf, false));
}

LK_DEVICE float lane_of(float v, int l) { return __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, v), l)); }

// grid (sequence, head), one wave: 64 tokens = 4 chunks per round.  pre: [T, H] of 4 floats
__global__ __launch_bounds__(64) void mlstm_gates_kernel(MlstmParams a, floatx4* __restrict__ pre) {
  const int s = blockIdx.x, h = blockIdx.y, lane = threadIdx.x;
  const int row0 = a.cu[s], len = a.cu[s + 1] - row0, slot = a.slots[s];
  if (len <= 0 || slot < 0) return;
  float m = a.positions[row0] == 0 ? 0.f : a.nm[((long)slot * a.H + h) * a.Z * (a.dk + 4) + a.dk];
  const float* gi = a.gates + (long)row0 * a.gs + h;
  float ni = -1e30f, nf = 0.f;
  if (lane < len) {
    ni = gi[(long)lane * a.gs];
    nf = gi[(long)lane * a.gs + a.H];
  }
  for (int t0 = 0; t0 < len; t0 += 64) {
    const float ig = ni;
    float F = nf;
    const int tn = t0 + 64 + lane;
    ni = -1e30f;
    nf = 0.f;
    if (tn < len) {   // the next round's gates travel under this round's scans
      ni = gi[(long)tn * a.gs];
      nf = gi[(long)tn * a.gs + a.H];
    }
    F += row_shr<1>(0.f, F);
    F += row_shr<2>(0.f, F);
    F += row_shr<4>(0.f, F);
    F += row_shr<8>(0.f, F);
    const float as = ig - F;
    float am = as;
    am = fmaxf(am, row_shr<1>(-1e30f, am));
    am = fmaxf(am, row_shr<2>(-1e30f, am));
    am = fmaxf(am, row_shr<4>(-1e30f, am));
    am = fmaxf(am, row_shr<8>(-1e30f, am));
    float min_ = m;
#pragma unroll
    for (int c = 0; c < 4; ++c) {
      if ((lane >> 4) == c) min_ = m;
      m = lane_of(F, 16 * c + 15) + fmaxf(m, lane_of(am, 16 * c + 15));
    }
    const float mt = F + fmaxf(min_, am);
    if (t0 + lane < len) pre[(long)(row0 + t0 + lane) * a.H + h] = floatx4{as, F - mt, F - mt + min_, mt};
  }
}

// grid (sequence, head, column block): wave w owns the 16 state columns j0 + 16 w .. + 15 (all dk rows: NR accumulator tiles).
// Tokens past the end of the last chunk get a = -1e30 and the last token's c, m: they neither decay nor feed the state.
// VEC: 16-byte pieces of q and k rows, 4 adjacent columns of v (host check).
template <typename T, int NR, bool VEC>
__global__ __launch_bounds__(256) void mlstm_chunk_kernel(MlstmParams a, const floatx4* __restrict__ pre) {
  constexpr int NP = NR * 16, LD = NP + 4, L = kChunk, EV = 16 / sizeof(T), LH = NP + 8;
  constexpr bool BF = sizeof(T) == 2 && NP % 32 == 0;
  __shared__ __attribute__((aligned(16))) float sk[L][LD];
  __shared__ __attribute__((aligned(16))) float sq[L][LD];
  __shared__ __attribute__((aligned(16))) bf16_t hk[BF ? L : 1][BF ? LH : 8];   // the raw bf16 rows (q.k products)
  __shared__ __attribute__((aligned(16))) bf16_t hq[BF ? L : 1][BF ? LH : 8];
  __shared__ __attribute__((aligned(16))) float sv[L][kColBlock + 4], sn[2][NP];
  __shared__ __attribute__((aligned(16))) float ga[L], gc[L], ge[L], gw[L], gm[L];   // a_s, c_t, e_t, D_Ls, exp(-m_t)
  const int s = blockIdx.x, h = blockIdx.y, z = blockIdx.z, tid = threadIdx.x, j0 = z * kColBlock;
  const int lane = tid & 63, w = tid >> 6, n16 = lane & 15, g = lane >> 4;
  const int col = j0 + 16 * w + n16;
  const bool cv = col < a.dv;
  const int row0 = a.cu[s], len = a.cu[s + 1] - row0, slot = a.slots[s];
  if (len <= 0) return;
  if (slot < 0) {
    zero_rows(a, row0, len, h, j0, 256);
    return;
  }
  auto ex = [](float x) {   // accurate exponential for f32 rows, the hardware one for bf16 rows (whose own rounding is 2^-9)
    if constexpr (sizeof(T) == 4) return expf(x);
    else return __expf(x);
  };
  const bool fresh = a.positions[row0] == 0;
  float* Sg = a.S + ((long)slot * a.H + h) * a.dk * a.dv + (cv ? col : 0);
  float* nmg = a.nm + (((long)slot * a.H + h) * a.Z + z) * (a.dk + 4);
  floatx4 S[NR];
#pragma unroll
  for (int nt = 0; nt < NR; ++nt) S[nt] = floatx4{0.f, 0.f, 0.f, 0.f};
  if (!fresh) {   // (loads from clamped places, selected afterwards: all in flight together)
#pragma unroll
    for (int nt = 0; nt < NR; ++nt)
#pragma unroll
      for (int j = 0; j < 4; ++j) S[nt][j] = Sg[(long)min(nt * 16 + 4 * g + j, a.dk - 1) * a.dv];
#pragma unroll
    for (int nt = 0; nt < NR; ++nt)
#pragma unroll
      for (int j = 0; j < 4; ++j) S[nt][j] = cv && nt * 16 + 4 * g + j < a.dk ? S[nt][j] : 0.f;
  }
  for (int i = tid; i < NP; i += 256) sn[0][i] = (!fresh && i < a.dk) ? nmg[i] : 0.f;
  const T* qg = reinterpret_cast<const T*>(a.q) + (long)h * a.dk;
  const T* kg = reinterpret_cast<const T*>(a.k) + (long)h * a.dk;
  const T* vg = reinterpret_cast<const T*>(a.v) + (long)h * a.dv;
  // The next chunk's operands are requested before this chunk's products are issued, as raw pieces from clamped places: nothing
  // is converted, masked or branched on until they are staged, so no load is waited for here.
  constexpr int CPR = NP / EV, NPF = (2 * L * CPR + 255) / 256;
  const int vt = tid >> 4, vc = j0 + 4 * (tid & 15);   // this thread's token and first of 4 columns of v
  uint4_t stg[NPF];
  T stv[4];
  floatx4 gt0, gl0;   // this token's and the chunk's last token's gate terms
  auto fetch = [&](int t0) {
    const int tl = min(L, len - t0), ncpr = a.dk / EV;
    if constexpr (VEC) {
#pragma unroll
      for (int x = 0; x < NPF; ++x) {
        const int i = min(tid + 256 * x, 2 * L * CPR - 1);
        const int which = i / (L * CPR), r = i % (L * CPR), t = min(r / CPR, tl - 1), c = min(r % CPR, ncpr - 1);
        const T* src = which ? qg : kg;
        stg[x] = *reinterpret_cast<const uint4_t*>(src + (long)(row0 + t0 + t) * (which ? a.qs : a.ks) + c * EV);
      }
    }
    const T* vr = vg + (long)(row0 + t0 + min(vt, tl - 1)) * a.vs;
    if constexpr (VEC) {
      if constexpr (sizeof(T) == 2) *reinterpret_cast<short4_t*>(stv) = *reinterpret_cast<const short4_t*>(vr + min(vc, a.dv - 4));
      else *reinterpret_cast<floatx4*>(stv) = *reinterpret_cast<const floatx4*>(vr + min(vc, a.dv - 4));
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e) stv[e] = vr[min(vc + e, a.dv - 1)];
    }
    gl0 = pre[(long)(row0 + t0 + tl - 1) * a.H + h];
    gt0 = pre[(long)(row0 + t0 + min(n16, tl - 1)) * a.H + h];
  };
  fetch(0);
  int cur = 0;
  for (int t0 = 0; t0 < len; t0 += L) {
    const int tl = min(L, len - t0);
    __syncthreads();   // the previous chunk has been consumed
    if constexpr (VEC) {
#pragma unroll
      for (int x = 0; x < NPF; ++x) {
        const int i = tid + 256 * x;
        if (i < 2 * L * CPR) {
          const int which = i / (L * CPR), r = i % (L * CPR), t = r / CPR, c = r % CPR;
          float* dst = (which ? sq[t] : sk[t]) + c * EV;
          const float f = which ? a.q_scale : 1.f;
          if (t >= tl || c >= a.dk / EV) stg[x] = uint4_t{0u, 0u, 0u, 0u};
          if constexpr (sizeof(T) == 2) {
            const short8 v = __builtin_bit_cast(short8, stg[x]);
            *reinterpret_cast<floatx4*>(dst) = floatx4{bf2f((bf16_t)v[0]) * f, bf2f((bf16_t)v[1]) * f, bf2f((bf16_t)v[2]) * f, bf2f((bf16_t)v[3]) * f};
            *reinterpret_cast<floatx4*>(dst + 4) = floatx4{bf2f((bf16_t)v[4]) * f, bf2f((bf16_t)v[5]) * f, bf2f((bf16_t)v[6]) * f, bf2f((bf16_t)v[7]) * f};
            if constexpr (BF) *reinterpret_cast<uint4_t*>((which ? hq[t] : hk[t]) + c * EV) = stg[x];
          } else {
            const floatx4 v = __builtin_bit_cast(floatx4, stg[x]);
            *reinterpret_cast<floatx4*>(dst) = floatx4{v[0] * f, v[1] * f, v[2] * f, v[3] * f};
          }
        }
      }
    } else {
      for (int i = tid; i < 2 * L * NP; i += 256) {
        const int which = i / (L * NP), r = i % (L * NP), t = r / NP, c = r % NP;
        const bool in = t < tl && c < a.dk;
        const long row = row0 + t0 + t;
        T raw = T(0);
        if (in) raw = which ? qg[row * a.qs + c] : kg[row * a.ks + c];
        (which ? sq[t] : sk[t])[c] = ldf<T>(&raw) * (which ? a.q_scale : 1.f);
        if constexpr (BF) (which ? hq[t] : hk[t])[c] = raw;
      }
    }
    {
      floatx4 v;
#pragma unroll
      for (int e = 0; e < 4; ++e) v[e] = vt < tl && vc + e < a.dv ? ldf<T>(stv + e) : 0.f;
      *reinterpret_cast<floatx4*>(&sv[vt][vc - j0]) = v;
    }
    {   // (every thread evaluates its token's terms, 16 of them store: no load is left in flight on a path that skips its use)
      const bool in = n16 < tl;
      const float as = in ? gt0[0] : -1e30f, cc = in ? gt0[1] : gl0[1], ee = ex(in ? gt0[2] : gl0[2]), mm = ex(in ? -gt0[3] : -gl0[3]),
                  ww = ex(gl0[1] + as);
      if (tid < L) {
        ga[tid] = as;
        gc[tid] = cc;
        ge[tid] = ee;
        gm[tid] = mm;
        gw[tid] = ww;
      }
    }
    __syncthreads();
    if (t0 + L < len) fetch(t0 + L);
    // G^T: lane (t = n16, g) gets G[t][s = 4g + j] = q_t . k_s
    floatx4 gt = {0.f, 0.f, 0.f, 0.f};
    if constexpr (BF) {
#pragma unroll
      for (int nb = 0; nb < NP / 32; ++nb) {
        const short8 ka = *reinterpret_cast<const short8*>(&hk[n16][nb * 32 + 8 * g]);
        const short8 qb = *reinterpret_cast<const short8*>(&hq[n16][nb * 32 + 8 * g]);
        gt = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ka, qb, gt, 0, 0, 0);
      }
#pragma unroll
      for (int j = 0; j < 4; ++j) gt[j] *= a.q_scale;
    } else {
#pragma unroll
      for (int nb = 0; nb < NR; ++nb) {
        const floatx4 a4 = *reinterpret_cast<const floatx4*>(&sk[n16][nb * 16 + 4 * g]);
        const floatx4 b4 = *reinterpret_cast<const floatx4*>(&sq[n16][nb * 16 + 4 * g]);
#pragma unroll
        for (int j = 0; j < 4; ++j) gt = __builtin_amdgcn_mfma_f32_16x16x4f32(a4[j], b4[j], gt, 0, 0, 0);
      }
    }
    // num: rows t = 4g + j, column n16 of this wave's tile; n . q of t = n16 beside it
    floatx4 ya = {0.f, 0.f, 0.f, 0.f};
    float nq = 0.f;
#pragma unroll
    for (int nt = 0; nt < NR; ++nt) {
      const floatx4 q4 = *reinterpret_cast<const floatx4*>(&sq[n16][nt * 16 + 4 * g]);
      const floatx4 n4 = *reinterpret_cast<const floatx4*>(&sn[cur][nt * 16 + 4 * g]);
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        ya = __builtin_amdgcn_mfma_f32_16x16x4f32(q4[j], S[nt][j], ya, 0, 0, 0);
        nq += q4[j] * n4[j];
      }
    }
    const floatx4 a4 = *reinterpret_cast<const floatx4*>(&ga[4 * g]), e4 = *reinterpret_cast<const floatx4*>(&ge[4 * g]),
                  w4 = *reinterpret_cast<const floatx4*>(&gw[4 * g]);
    const float ct = gc[n16];
    float M[4], xv[4];
    nq *= ge[n16];   // (each lane group holds its quarter of both sums of t = n16)
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      M[j] = 4 * g + j <= n16 ? gt[j] * ex(ct + a4[j]) : 0.f;
      nq += M[j];
      xv[j] = sv[4 * g + j][16 * w + n16];
    }
    nq += __shfl_xor(nq, 16, 64);
    nq += __shfl_xor(nq, 32, 64);
    const float rden = 1.f / (fmaxf(fabsf(nq), gm[n16]) + kDenEps);
#pragma unroll
    for (int j = 0; j < 4; ++j) ya[j] *= e4[j];
#pragma unroll
    for (int j = 0; j < 4; ++j) ya = __builtin_amdgcn_mfma_f32_16x16x4f32(M[j], xv[j], ya, 0, 0, 0);
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int t = 4 * g + j;
      const float rd = __shfl(rden, t, 16);
      if (cv && t < tl) a.o[(long)(row0 + t0 + t) * a.os + (long)h * a.dv + col] = ya[j] * rd;
    }
    // state: rows i = 16 nt + 4g + j, column n16
    const float dec = ge[L - 1];
#pragma unroll
    for (int j = 0; j < 4; ++j) xv[j] *= w4[j];   // D_Ls v_s
#pragma unroll
    for (int nt = 0; nt < NR; ++nt) {
#pragma unroll
      for (int j = 0; j < 4; ++j) S[nt][j] *= dec;
    }
#pragma unroll
    for (int j = 0; j < 4; ++j)
#pragma unroll
      for (int nt = 0; nt < NR; ++nt) S[nt] = __builtin_amdgcn_mfma_f32_16x16x4f32(sk[4 * g + j][nt * 16 + n16], xv[j], S[nt], 0, 0, 0);
    // n: a wave owns NP / 4 of its entries, PARTS lanes share one and take 16 / PARTS tokens each
    constexpr int NW = NP / 4, PARTS = 64 / NW;
    {
      const int i = w * NW + lane % NW, part = lane / NW;
      float v = 0.f;
#pragma unroll
      for (int x = 0; x < L / PARTS; ++x) v += gw[part * (L / PARTS) + x] * sk[part * (L / PARTS) + x][i];
#pragma unroll
      for (int d = NW; d < 64; d <<= 1) v += __shfl_xor(v, d, 64);
      if (part == 0) sn[cur ^ 1][i] = dec * sn[cur][i] + v;
    }
    cur ^= 1;
  }
  __syncthreads();
  if (cv) {
#pragma unroll
    for (int nt = 0; nt < NR; ++nt)
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int i = nt * 16 + 4 * g + j;
        if (i < a.dk) Sg[(long)i * a.dv] = S[nt][j];
      }
  }
  for (int i = tid; i < a.dk; i += 256) nmg[i] = sn[cur][i];
  if (tid == 0) nmg[a.dk] = pre[(long)(row0 + len - 1) * a.H + h][3];
}

template <typename T>
int scan_t(const MlstmParams& a, int S, int max_len, floatx4* pre, hipStream_t st) {
  const dim3 grid((unsigned)S, (unsigned)a.H, (unsigned)a.Z);
  if (max_len >= kChunkMin) {
    if (!pre) return -1;
    mlstm_gates_kernel<<<dim3((unsigned)S, (unsigned)a.H), 64, 0, st>>>(a, pre);
    LK_CHECK_LAUNCH();
    constexpr int ev = 16 / (int)sizeof(T);
    const auto al = [](const void* x, int b) { return reinterpret_cast<uintptr_t>(x) % b == 0; };
    const bool cvec = a.dk % ev == 0 && a.qs % ev == 0 && a.ks % ev == 0 && al(a.q, 16) && al(a.k, 16) && a.dv % 4 == 0 && a.vs % 4 == 0 &&
                      al(a.v, 4 * sizeof(T));
#define LK_CHUNK(NR)                                                         \
  if (cvec) mlstm_chunk_kernel<T, NR, true><<<grid, 256, 0, st>>>(a, pre);    \
  else mlstm_chunk_kernel<T, NR, false><<<grid, 256, 0, st>>>(a, pre)
    if (a.dk <= 16) { LK_CHUNK(1); }
    else if (a.dk <= 32) { LK_CHUNK(2); }
    else if (a.dk <= 64) { LK_CHUNK(4); }
    else if (a.dk <= 128) { LK_CHUNK(8); }
    else if (a.dk <= 256) { LK_CHUNK(16); }
    else return -1;
#undef LK_CHUNK
  } else {
    const bool vec = a.dv % 4 == 0 && reinterpret_cast<uintptr_t>(a.S) % 16 == 0;
#define LK_STEP(NR)                                               \
  if (vec) mlstm_step_kernel<T, NR, true><<<grid, 256, 0, st>>>(a); \
  else mlstm_step_kernel<T, NR, false><<<grid, 256, 0, st>>>(a)
    if (a.dk <= 16) { LK_STEP(1); }
    else if (a.dk <= 32) { LK_STEP(2); }
    else if (a.dk <= 64) { LK_STEP(4); }
    else if (a.dk <= 128) { LK_STEP(8); }
    else if (a.dk <= 256) { LK_STEP(16); }
    else return -1;
#undef LK_STEP
  }
  LK_CHECK_LAUNCH();
  return 0;
}

}  // namespace

// the chunked form runs when some sequence of the step has this many rows: it needs `pre`, [rows, H, 4] f32 scratch
int lk_mlstm_chunk_min() { return kChunkMin; }

int lk_mlstm_scan(const void* q, long qs, const void* k, long ks, const void* v, long vs, int esz, const float* gates, long gs, float q_scale,
                  float* S, float* nm, const int* cu, const int* slots, const int* positions, int seqs, int H, int dk, int dv, float* o,
                  long os, int max_len, float* pre, hipStream_t st) {
  if (seqs <= 0) return 0;
  if (H < 1 || H > 65535 || dk < 1 || dk > 256 || dv < 1 || (dv + kColBlock - 1) / kColBlock > 65535) return -1;
  MlstmParams a;
  a.q = q; a.k = k; a.v = v; a.qs = qs; a.ks = ks; a.vs = vs; a.gates = gates; a.gs = gs; a.q_scale = q_scale; a.S = S; a.nm = nm;
  a.cu = cu; a.slots = slots; a.positions = positions; a.o = o; a.os = os; a.H = H; a.dk = dk; a.dv = dv;
  a.Z = (dv + kColBlock - 1) / kColBlock;
  return esz == 2 ? scan_t<bf16_t>(a, seqs, max_len, reinterpret_cast<floatx4*>(pre), st)
                  : scan_t<float>(a, seqs, max_len, reinterpret_cast<floatx4*>(pre), st);
}
