// Gated delta rule with one decay per head and token.  Per head and sequence, from the convolutions' q, k, v and two raw numbers a_t, b_t:
//
//   g_t = exp(-exp(A) softplus(a_t + dt)),  beta_t = sigmoid(b_t),  k^_t = k_t rk_t,  q^_t = q_t rq_t
//   rk_t = 1 / sqrt(|k_t|^2 + 1e-6),  rq_t = dk^(-1/2) / sqrt(|q_t|^2 + 1e-6)
//   S <- g_t S;  u_t = beta_t (v_t - S^T k^_t);  S <- S + k^_t u_t^T;  o_t = S^T q^_t            S [dk, dv] f32
//   out_t = o_t / sqrt(mean(o_t^2) + eps) * w * silu(gate_t)
//
// A batch is a list of sequences (prompt portions of any length, decode rows of length 1): rows [cu[s], cu[s+1]) belong to sequence s,
// whose state lives in slot slots[s] (< 0: a padding row, its output rows are zero) and starts from zero when its first row
// sits at position 0.
//
// Steps of single tokens: one workgroup per (sequence, head) streams the state once and finishes the row (norm and gate included).
//
// Steps with longer portions run in chunks of 16 tokens.  With G_t = ln g_1 + .. + ln g_t inside the chunk and S the state in front of it,
//   (I + A) U = diag(beta) (V - diag(e^G) K^ S),    A_ts = beta_t e^(G_t - G_s) k^_t.k^_s  (s < t)
//   O = diag(e^G) Q^ S + P U,                       P_ts = e^(G_t - G_s) q^_t.k^_s         (s <= t)
//   S' = e^(G_L) S + sum_s e^(G_L - G_s) k^_s u_s^T
// Nothing of B = (I + A)^(-1) diag(beta), P and the row factors depends on S: a kernel of one wave per (chunk, head) makes them first, for
// all chunks at once; the chain from chunk to chunk is three products with the state in MFMA accumulators.  All products that touch
// the state are f32.  The running sums G are f64: their differences must keep f32 accuracy behind a large decay.
#include "common.h"
#include "kernels.h"
#include "attn_frag.h"

namespace {

constexpr float kUnitEps = 1e-6f;
constexpr int kL = 16;       // tokens of a chunk
constexpr int kPre = 36;     // f32 of a (token, head) that the chunk kernel reads: a row of B, a row of P, 4 row factors

LK_DEVICE float sigmoid_f(float x) { return 1.f / (1.f + expf(-x)); }
LK_DEVICE float softplus_f(float x) { return x > 20.f ? x : log1pf(expf(x)); }

struct HeadDeltaParams {
  const void* q;   // rows of Hk * dk
  const void* k;
  const void* v;   // rows of H * dv
  const void* b;   // rows of H
  const void* a;
  const void* gate;  // rows of H * dv
  long qs, ks, vs, bs, as, gs;
  const float* dt_bias;
  const float* A_log;
  const float* norm_w;
  float eps;
  float* state;  // [slots, H, dk, dv]
  const int* cu;
  const int* slots;
  const int* positions;
  int H, Hk, dk, dv;
  void* out;
  long os;
  float* pre;   // [rows, H, kPre]
  float* o;     // [rows, H * dv]
};

// ---- single tokens.  512 (256) threads = 32 (16) groups of 4 adjacent state columns x 16 row slices; a thread holds the rows rs,
// rs + 16, ... of its 4 columns (16-byte accesses, VEC), and the workgroup walks the head's columns in blocks of 128 (64).
template <typename T, int NR, int CGN, bool VEC>
__global__ __launch_bounds__(16 * CGN, NR <= 8 ? 4 : 2) void head_delta_step_kernel(HeadDeltaParams p) {
  constexpr int NT = 16 * CGN, NW = NT / 64, COLS = 4 * CGN;
  __shared__ float sq[NR * 16], sk[NR * 16], red[NW][CGN][9], so[1024];
  const int s = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int row = p.cu[s], len = p.cu[s + 1] - row, slot = p.slots[s];
  if (len <= 0) return;
  T* orow = reinterpret_cast<T*>(p.out) + (long)row * p.os + (long)h * p.dv;
  if (slot < 0) {
    for (int c = tid; c < p.dv; c += NT) El<T>::st(orow + c, 0.f);
    return;
  }
  const int cg = tid % CGN, rs = tid / CGN, wv = tid >> 6, lane = tid & 63;
  const bool fresh = p.positions[row] == 0;
  float* Sh = p.state + ((long)slot * p.H + h) * p.dk * p.dv;
  floatx4 S[NR];
  auto load_state = [&](int c0) {
#pragma unroll
    for (int ii = 0; ii < NR; ++ii) {
      const int i = rs + 16 * ii;
      S[ii] = floatx4{0.f, 0.f, 0.f, 0.f};
      if (!fresh && i < p.dk) {
        const float* src = Sh + (long)i * p.dv + c0;
        if constexpr (VEC) {
          if (c0 < p.dv) S[ii] = *reinterpret_cast<const floatx4*>(src);
        } else {
#pragma unroll
          for (int e = 0; e < 4; ++e)
            if (c0 + e < p.dv) S[ii][e] = src[e];
        }
      }
    }
  };
  load_state(4 * cg);
  const int kh = h / (p.H / p.Hk);
  if (wv < 2) {   // wave 0: the unit query times dk^(-1/2), wave 1: the unit key
    const T* x = wv == 0 ? reinterpret_cast<const T*>(p.q) + (long)row * p.qs + (long)kh * p.dk
                         : reinterpret_cast<const T*>(p.k) + (long)row * p.ks + (long)kh * p.dk;
    float* dst = wv == 0 ? sq : sk;
    float e[NR > 4 ? NR / 4 : 1], ss = 0.f;
#pragma unroll
    for (int i = 0; i < (NR > 4 ? NR / 4 : 1); ++i) {
      const int c = lane + 64 * i;
      e[i] = c < p.dk ? El<T>::ld(x + c) : 0.f;
      ss += e[i] * e[i];
    }
    const float inv = (1.f / sqrtf(wave_sum(ss) + kUnitEps)) * (wv == 0 ? 1.f / sqrtf((float)p.dk) : 1.f);
#pragma unroll
    for (int i = 0; i < (NR > 4 ? NR / 4 : 1); ++i)
      if (lane + 64 * i < NR * 16) dst[lane + 64 * i] = e[i] * inv;
  }
  const float beta = sigmoid_f(El<T>::ld(reinterpret_cast<const T*>(p.b) + (long)row * p.bs + h));
  const float dec = expf(-expf(p.A_log[h]) * softplus_f(El<T>::ld(reinterpret_cast<const T*>(p.a) + (long)row * p.as + h) + p.dt_bias[h]));
  __syncthreads();
  for (int j0 = 0; j0 < p.dv; j0 += COLS) {
    const int c0 = j0 + 4 * cg;
    float v[4], acc[9];
#pragma unroll
    for (int e = 0; e < 4; ++e)
      v[e] = c0 + e < p.dv ? El<T>::ld(reinterpret_cast<const T*>(p.v) + (long)row * p.vs + (long)h * p.dv + c0 + e) : 0.f;
#pragma unroll
    for (int e = 0; e < 9; ++e) acc[e] = 0.f;
#pragma unroll
    for (int ii = 0; ii < NR; ++ii) {
      const float kk = sk[rs + 16 * ii], qq = sq[rs + 16 * ii];
      acc[8] += kk * qq;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        acc[e] += kk * S[ii][e];
        acc[4 + e] += qq * S[ii][e];
      }
    }
#pragma unroll
    for (int e = 0; e < 9; ++e) {
      if constexpr (CGN == 16) acc[e] += __shfl_xor(acc[e], 16, 64);
      acc[e] += __shfl_xor(acc[e], 32, 64);
    }
    if (lane < CGN) {
#pragma unroll
      for (int e = 0; e < 9; ++e) red[wv][lane][e] = acc[e];
    }
    __syncthreads();
#pragma unroll
    for (int e = 0; e < 9; ++e) {
      float t = 0.f;
#pragma unroll
      for (int i = 0; i < NW; ++i) t += red[i][cg][e];
      acc[e] = t;
    }
    float u[4];
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      u[e] = beta * (v[e] - dec * acc[e]);
      if (rs == 0 && c0 + e < p.dv) so[c0 + e] = dec * acc[4 + e] + acc[8] * u[e];
    }
#pragma unroll
    for (int ii = 0; ii < NR; ++ii) {
      const int i = rs + 16 * ii;
      if (i < p.dk) {
        const float kk = sk[i];
#pragma unroll
        for (int e = 0; e < 4; ++e) S[ii][e] = dec * S[ii][e] + kk * u[e];
        float* dst = Sh + (long)i * p.dv + c0;
        if constexpr (VEC) {
          if (c0 < p.dv) *reinterpret_cast<floatx4*>(dst) = S[ii];
        } else {
#pragma unroll
          for (int e = 0; e < 4; ++e)
            if (c0 + e < p.dv) dst[e] = S[ii][e];
        }
      }
    }
    if (j0 + COLS < p.dv) load_state(c0 + COLS);
    __syncthreads();   // sums read, this block's outputs written
  }
  if (wv == 0) {
    float ss = 0.f;
    for (int c = lane; c < p.dv; c += 64) ss += so[c] * so[c];
    const float inv = 1.f / sqrtf(wave_sum(ss) / (float)p.dv + p.eps);
    const T* gr = reinterpret_cast<const T*>(p.gate) + (long)row * p.gs + (long)h * p.dv;
    for (int c = lane; c < p.dv; c += 64) {
      const float gv = El<T>::ld(gr + c);
      El<T>::st(orow + c, so[c] * inv * p.norm_w[(long)h * p.dv + c] * (gv * sigmoid_f(gv)));
    }
  }
}

// ---- chunk operands: one wave per (chunk, head), grid (chunks of the longest sequence, heads / 4, sequences)
template <typename T>
__global__ __launch_bounds__(256) void head_delta_chunk_pre_kernel(HeadDeltaParams p, bool vec) {
  constexpr int EV = El<T>::V, KF = 4 * EV;   // contraction of one fragment step
  __shared__ __attribute__((aligned(16))) float sA[4][kL][kL + 4];
  const int s = blockIdx.z, w = threadIdx.x >> 6, lane = threadIdx.x & 63, n16 = lane & 15, g = lane >> 4;
  const int h = blockIdx.y * 4 + w, t0 = blockIdx.x * kL;
  const int row0 = p.cu[s], len = p.cu[s + 1] - row0;
  if (t0 >= len || p.slots[s] < 0 || h >= p.H) return;   // (no barrier below: a wave works alone)
  const int tl = min(kL, len - t0), kh = h / (p.H / p.Hk);
  const long row = row0 + t0 + min(n16, tl - 1);
  const T* kr = reinterpret_cast<const T*>(p.k) + row * p.ks + (long)kh * p.dk;
  const T* qr = reinterpret_cast<const T*>(p.q) + row * p.qs + (long)kh * p.dk;
  floatx4 kk = {0.f, 0.f, 0.f, 0.f}, qk = {0.f, 0.f, 0.f, 0.f};   // [s = 4g + j][t = n16]
  float ssk = 0.f, ssq = 0.f;
  for (int d = 0; d < p.dk; d += KF) {
    const uint4_t kf = frag<T>(kr, d + g * EV, p.dk, vec), qf = frag<T>(qr, d + g * EV, p.dk, vec);
    kk = mma_qk<T>(kf, kf, kk);
    qk = mma_qk<T>(kf, qf, qk);
    const T *ke = reinterpret_cast<const T*>(&kf), *qe = reinterpret_cast<const T*>(&qf);
#pragma unroll
    for (int e = 0; e < EV; ++e) {
      const float x = El<T>::ld(ke + e), y = El<T>::ld(qe + e);
      ssk += x * x;
      ssq += y * y;
    }
  }
  ssk += __shfl_xor(ssk, 16, 64);
  ssk += __shfl_xor(ssk, 32, 64);
  ssq += __shfl_xor(ssq, 16, 64);
  ssq += __shfl_xor(ssq, 32, 64);
  const float rk = 1.f / sqrtf(ssk + kUnitEps), rq = (1.f / sqrtf(ssq + kUnitEps)) * (1.f / sqrtf((float)p.dk));
  const bool in = n16 < tl;
  const float beta = in ? sigmoid_f(El<T>::ld(reinterpret_cast<const T*>(p.b) + row * p.bs + h)) : 0.f;
  const float la = in ? -expf(p.A_log[h]) * softplus_f(El<T>::ld(reinterpret_cast<const T*>(p.a) + row * p.as + h) + p.dt_bias[h]) : 0.f;
  double G = la;
#pragma unroll
  for (int d = 1; d < kL; d <<= 1) {
    const double o = __shfl_up(G, d, kL);
    if (n16 >= d) G += o;
  }
  const double GL = __shfl(G, tl - 1, kL);
  floatx4 P;
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int sj = 4 * g + j;
    const float dec = sj <= n16 ? expf((float)(G - __shfl(G, sj, kL))) : 0.f, rs = __shfl(rk, sj, kL);
    P[j] = dec * rq * rs * qk[j];
    sA[w][n16][sj] = sj < n16 ? beta * dec * rk * rs * kk[j] : 0.f;
  }
  // column n16 of (I + A)^(-1) by forward substitution (every lane group alike), LDS of this wave only
  __builtin_amdgcn_wave_barrier();
  float x[kL];
#pragma unroll
  for (int t = 0; t < kL; ++t) {
    float v = t == n16 ? 1.f : 0.f;
#pragma unroll
    for (int c = 0; c < t; c += 4) {
      const floatx4 ar = *reinterpret_cast<const floatx4*>(&sA[w][t][c]);
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (c + e < t) v -= ar[e] * x[c + e];
    }
    x[t] = v;
  }
  float* dst = p.pre + ((long)(row0 + t0) * p.H + h) * kPre;
  const long st = (long)p.H * kPre;
#pragma unroll
  for (int j = 0; j < 4; ++j) {   // B row t = 4g + j, column n16
    const float v = g == 0 ? x[j] : g == 1 ? x[4 + j] : g == 2 ? x[8 + j] : x[12 + j];
    if (4 * g + j < tl) dst[(4 * g + j) * st + n16] = v * beta;
  }
  if (in) {
    *reinterpret_cast<floatx4*>(dst + n16 * st + 16 + 4 * g) = P;
    if (g == 0) {
      const float et = expf((float)G);
      *reinterpret_cast<floatx4*>(dst + n16 * st + 32) = floatx4{et * rk, et * rq, rk * expf((float)(GL - G)), expf((float)GL)};
    }
  }
}

// ---- the chain over the chunks: grid (sequence, head, block of 16 NW state columns), wave w owns 16 of them (all dk rows: NR
// accumulator tiles).  VEC: 16-byte pieces of q and k rows, 4 adjacent columns of v (host check).
template <typename T, int NR, int NW, bool VEC>
__global__ __launch_bounds__(64 * NW) void head_delta_chunk_kernel(HeadDeltaParams p) {
  constexpr int NP = NR * 16, LD = NP + 4, EV = El<T>::V, NT = 64 * NW, COLS = 16 * NW;
  constexpr int NB = NR <= 8 ? 2 : 1;   // LDS buffers (two: one barrier per chunk)
  __shared__ __attribute__((aligned(16))) float sk[NB][kL][LD];
  __shared__ __attribute__((aligned(16))) float sq[NB][kL][LD];
  __shared__ __attribute__((aligned(16))) float sv[NB][kL][COLS + 4];
  __shared__ __attribute__((aligned(16))) float sp[NB][kL][kPre];
  const int s = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, j0 = blockIdx.z * COLS;
  const int lane = tid & 63, w = tid >> 6, n16 = lane & 15, g = lane >> 4;
  const int col = j0 + 16 * w + n16;
  const bool cv = col < p.dv;
  const int row0 = p.cu[s], len = p.cu[s + 1] - row0, slot = p.slots[s];
  if (len <= 0) return;
  float* og = p.o + (long)row0 * p.H * p.dv + (long)h * p.dv;
  if (slot < 0) {
    for (int i = tid; i < len * COLS; i += NT) {
      const int c = j0 + i % COLS;
      if (c < p.dv) og[(long)(i / COLS) * p.H * p.dv + c] = 0.f;
    }
    return;
  }
  const bool fresh = p.positions[row0] == 0;
  float* Sg = p.state + ((long)slot * p.H + h) * p.dk * p.dv + (cv ? col : 0);
  floatx4 S[NR];
#pragma unroll
  for (int nt = 0; nt < NR; ++nt) S[nt] = floatx4{0.f, 0.f, 0.f, 0.f};
  if (!fresh) {   // (loads from clamped places, selected afterwards: all in flight together)
#pragma unroll
    for (int nt = 0; nt < NR; ++nt)
#pragma unroll
      for (int j = 0; j < 4; ++j) S[nt][j] = Sg[(long)min(nt * 16 + 4 * g + j, p.dk - 1) * p.dv];
#pragma unroll
    for (int nt = 0; nt < NR; ++nt)
#pragma unroll
      for (int j = 0; j < 4; ++j) S[nt][j] = cv && nt * 16 + 4 * g + j < p.dk ? S[nt][j] : 0.f;
  }
  const int kh = h / (p.H / p.Hk);
  const T* qg = reinterpret_cast<const T*>(p.q) + (long)kh * p.dk;
  const T* kg = reinterpret_cast<const T*>(p.k) + (long)kh * p.dk;
  const T* vg = reinterpret_cast<const T*>(p.v) + (long)h * p.dv;
  const float* pg = p.pre + ((long)row0 * p.H + h) * kPre;
  // The next chunk's operands travel into registers under this chunk's products, as raw pieces from clamped places; they are
  // converted and masked as they are staged.
  constexpr int CPR = NP / EV, NQK = (2 * kL * CPR + NT - 1) / NT, NV = (kL * COLS / 4 + NT - 1) / NT, NPR = (kL * kPre / 4 + NT - 1) / NT;
  uint4_t rqk[NQK];
  T rv[NV][4];
  floatx4 rp[NPR];
  auto fetch = [&](int t0) {
    const int tl = min(kL, len - t0), ncpr = p.dk / EV;
    if constexpr (VEC) {
#pragma unroll
      for (int x = 0; x < NQK; ++x) {
        const int i = min(tid + NT * x, 2 * kL * CPR - 1), which = i / (kL * CPR), r = i % (kL * CPR);
        const int t = min(r / CPR, tl - 1), c = min(r % CPR, ncpr - 1);
        rqk[x] = ld16((which ? qg : kg) + (long)(row0 + t0 + t) * (which ? p.qs : p.ks) + c * EV);
      }
    }
#pragma unroll
    for (int x = 0; x < NV; ++x) {
      const int i = min(tid + NT * x, kL * COLS / 4 - 1), t = min(i / (COLS / 4), tl - 1), c = j0 + 4 * (i % (COLS / 4));
      const T* vr = vg + (long)(row0 + t0 + t) * p.vs;
      if constexpr (VEC) {
        if constexpr (sizeof(T) == 2) *reinterpret_cast<short4_t*>(rv[x]) = *reinterpret_cast<const short4_t*>(vr + min(c, p.dv - 4));
        else *reinterpret_cast<floatx4*>(rv[x]) = *reinterpret_cast<const floatx4*>(vr + min(c, p.dv - 4));
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e) rv[x][e] = vr[min(c + e, p.dv - 1)];
      }
    }
#pragma unroll
    for (int x = 0; x < NPR; ++x) {
      const int i = min(tid + NT * x, kL * kPre / 4 - 1), t = min(i / (kPre / 4), tl - 1), c = i % (kPre / 4);
      rp[x] = *reinterpret_cast<const floatx4*>(pg + (long)(t0 + t) * p.H * kPre + 4 * c);
    }
  };
  auto stage = [&](int t0, int buf) {
    const int tl = min(kL, len - t0);
    if constexpr (VEC) {
#pragma unroll
      for (int x = 0; x < NQK; ++x) {
        const int i = tid + NT * x;
        if (2 * kL * CPR % NT == 0 || i < 2 * kL * CPR) {
          const int which = i / (kL * CPR), r = i % (kL * CPR), t = r / CPR, c = r % CPR;
          float* dst = (which ? sq[buf][t] : sk[buf][t]) + c * EV;
          const uint4_t raw = t >= tl || c >= p.dk / EV ? uint4_t{0u, 0u, 0u, 0u} : rqk[x];
          if constexpr (sizeof(T) == 2) {
            const short8 v = __builtin_bit_cast(short8, raw);
            *reinterpret_cast<floatx4*>(dst) = floatx4{bf2f((bf16_t)v[0]), bf2f((bf16_t)v[1]), bf2f((bf16_t)v[2]), bf2f((bf16_t)v[3])};
            *reinterpret_cast<floatx4*>(dst + 4) = floatx4{bf2f((bf16_t)v[4]), bf2f((bf16_t)v[5]), bf2f((bf16_t)v[6]), bf2f((bf16_t)v[7])};
          } else {
            *reinterpret_cast<floatx4*>(dst) = __builtin_bit_cast(floatx4, raw);
          }
        }
      }
    } else {
      for (int i = tid; i < 2 * kL * NP; i += NT) {
        const int which = i / (kL * NP), r = i % (kL * NP), t = r / NP, c = r % NP;
        const long row = row0 + t0 + t;
        float v = 0.f;
        if (t < tl && c < p.dk) v = El<T>::ld(which ? qg + row * p.qs + c : kg + row * p.ks + c);
        (which ? sq[buf][t] : sk[buf][t])[c] = v;
      }
    }
#pragma unroll
    for (int x = 0; x < NV; ++x) {
      const int i = tid + NT * x;
      if (kL * COLS / 4 % NT == 0 || i < kL * COLS / 4) {
        const int t = i / (COLS / 4), c = 4 * (i % (COLS / 4));
        floatx4 v;
#pragma unroll
        for (int e = 0; e < 4; ++e) v[e] = t < tl && j0 + c + e < p.dv ? El<T>::ld(rv[x] + e) : 0.f;
        *reinterpret_cast<floatx4*>(&sv[buf][t][c]) = v;
      }
    }
#pragma unroll
    for (int x = 0; x < NPR; ++x) {
      const int i = tid + NT * x;
      if (kL * kPre / 4 % NT == 0 || i < kL * kPre / 4) {
        const int t = i / (kPre / 4), c = i % (kPre / 4);
        floatx4 v = t < tl ? rp[x] : floatx4{0.f, 0.f, 0.f, 0.f};
        // (columns of B and P at or behind tl of a shorter last chunk: B's are beta = 0, P's are masked by s <= t < tl)
        *reinterpret_cast<floatx4*>(&sp[buf][t][4 * c]) = v;
      }
    }
  };
  fetch(0);
  stage(0, 0);
  if (kL < len) fetch(kL);
  __syncthreads();
  int cur = 0;
  for (int t0 = 0; t0 < len; t0 += kL) {
    const int tl = min(kL, len - t0);
    // K S and Q S: rows t = 4g + j, column n16 of this wave's tile
    floatx4 y1[2], y2[2];
#pragma unroll
    for (int x = 0; x < 2; ++x) y1[x] = y2[x] = floatx4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int nt = 0; nt < NR; ++nt) {
      const floatx4 k4 = *reinterpret_cast<const floatx4*>(&sk[cur][n16][nt * 16 + 4 * g]);
#pragma unroll
      for (int j = 0; j < 4; ++j) y1[nt & 1] = __builtin_amdgcn_mfma_f32_16x16x4f32(k4[j], S[nt][j], y1[nt & 1], 0, 0, 0);
    }
    float xv[4];
    floatx4 f4[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      f4[j] = *reinterpret_cast<const floatx4*>(&sp[cur][4 * g + j][32]);
      xv[j] = sv[cur][4 * g + j][16 * w + n16] - f4[j][0] * (y1[0][j] + y1[1][j]);
    }
#pragma unroll
    for (int nt = 0; nt < NR; ++nt) {
      const floatx4 q4 = *reinterpret_cast<const floatx4*>(&sq[cur][n16][nt * 16 + 4 * g]);
#pragma unroll
      for (int j = 0; j < 4; ++j) y2[nt & 1] = __builtin_amdgcn_mfma_f32_16x16x4f32(q4[j], S[nt][j], y2[nt & 1], 0, 0, 0);
    }
    floatx4 u = {0.f, 0.f, 0.f, 0.f}, o;
    const floatx4 b4 = *reinterpret_cast<const floatx4*>(&sp[cur][n16][4 * g]), p4 = *reinterpret_cast<const floatx4*>(&sp[cur][n16][16 + 4 * g]);
#pragma unroll
    for (int j = 0; j < 4; ++j) u = __builtin_amdgcn_mfma_f32_16x16x4f32(b4[j], xv[j], u, 0, 0, 0);
#pragma unroll
    for (int j = 0; j < 4; ++j) o[j] = f4[j][1] * (y2[0][j] + y2[1][j]);
#pragma unroll
    for (int j = 0; j < 4; ++j) o = __builtin_amdgcn_mfma_f32_16x16x4f32(p4[j], u[j], o, 0, 0, 0);
    // state: rows i = 16 nt + 4g + j, column n16
    const float dec = sp[cur][0][35];
#pragma unroll
    for (int nt = 0; nt < NR; ++nt)
#pragma unroll
      for (int j = 0; j < 4; ++j) S[nt][j] *= dec;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const float us = u[j] * f4[j][2];
#pragma unroll
      for (int nt = 0; nt < NR; ++nt) S[nt] = __builtin_amdgcn_mfma_f32_16x16x4f32(sk[cur][4 * g + j][nt * 16 + n16], us, S[nt], 0, 0, 0);
    }
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (cv && 4 * g + j < tl) og[(long)(t0 + 4 * g + j) * p.H * p.dv + col] = o[j];
    if (t0 + kL < len) {
      if constexpr (NB == 1) __syncthreads();   // this chunk has been consumed
      stage(t0 + kL, NB == 2 ? cur ^ 1 : 0);
      if (t0 + 2 * kL < len) fetch(t0 + 2 * kL);
      __syncthreads();
      cur = NB == 2 ? cur ^ 1 : 0;
    }
  }
  if (cv) {
#pragma unroll
    for (int nt = 0; nt < NR; ++nt)
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int i = nt * 16 + 4 * g + j;
        if (i < p.dk) Sg[(long)i * p.dv] = S[nt][j];
      }
  }
}

// The same chain for bf16 rows.  A bf16 row times the f32 state is exact as three bf16 products: the state is split into parts of 8
// mantissa bits (s = hi + mid + lo, each cut off, so the sum is s itself), and the MFMA sums the exact partial products in f32.  One
// 32-row step of the products with the state is then 3 MFMAs of 16 cycles instead of 8 of 32.
//
// LDS rows of q and k hold, per 32 channels, the order of the B operand that the state's accumulators give without a move: place 8 g + e
// is channel 4 g + e (e < 4) and 16 + 4 g + e - 4 (e >= 4).  The same rows read transposed (4 tokens x 16 channels at a time) feed
// the update; its B operand holds u's parts hi and mid of the same 4 tokens side by side, then lo beside zeros.
typedef short4_t __attribute__((address_space(3))) * lds_short4_ptr;

LK_DEVICE unsigned upper_halves(float a, float b) {   // bf16 cut-offs of a (low half) and b (high half)
  return __builtin_amdgcn_perm(__float_as_uint(b), __float_as_uint(a), 0x07060302u);
}
LK_DEVICE float cut(float v) { return __uint_as_float(__float_as_uint(v) & 0xffff0000u); }

template <int NR, int NW, bool VEC>
__global__ __launch_bounds__(64 * NW) void head_delta_chunk_bf16_kernel(HeadDeltaParams p) {
  static_assert(NR % 2 == 0, "32-row steps");
  constexpr int NP = NR * 16, NB = NR / 2, LH = NP + 24, NT = 64 * NW, COLS = 16 * NW;
  __shared__ __attribute__((aligned(16))) bf16_t hk[2][kL][LH];
  __shared__ __attribute__((aligned(16))) bf16_t hq[2][kL][LH];
  __shared__ __attribute__((aligned(16))) float sv[2][kL][COLS + 4];
  __shared__ __attribute__((aligned(16))) float sp[2][kL][kPre];
  const int s = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, j0 = blockIdx.z * COLS;
  const int lane = tid & 63, w = tid >> 6, n16 = lane & 15, g = lane >> 4;
  const int col = j0 + 16 * w + n16;
  const bool cv = col < p.dv;
  const int row0 = p.cu[s], len = p.cu[s + 1] - row0, slot = p.slots[s];
  if (len <= 0) return;
  float* og = p.o + (long)row0 * p.H * p.dv + (long)h * p.dv;
  if (slot < 0) {
    for (int i = tid; i < len * COLS; i += NT) {
      const int c = j0 + i % COLS;
      if (c < p.dv) og[(long)(i / COLS) * p.H * p.dv + c] = 0.f;
    }
    return;
  }
  const bool fresh = p.positions[row0] == 0;
  float* Sg = p.state + ((long)slot * p.H + h) * p.dk * p.dv + (cv ? col : 0);
  floatx4 S[NR];
#pragma unroll
  for (int nt = 0; nt < NR; ++nt) S[nt] = floatx4{0.f, 0.f, 0.f, 0.f};
  if (!fresh) {   // (loads from clamped places, selected afterwards: all in flight together)
#pragma unroll
    for (int nt = 0; nt < NR; ++nt)
#pragma unroll
      for (int j = 0; j < 4; ++j) S[nt][j] = Sg[(long)min(nt * 16 + 4 * g + j, p.dk - 1) * p.dv];
#pragma unroll
    for (int nt = 0; nt < NR; ++nt)
#pragma unroll
      for (int j = 0; j < 4; ++j) S[nt][j] = cv && nt * 16 + 4 * g + j < p.dk ? S[nt][j] : 0.f;
  }
  const int kh = h / (p.H / p.Hk);
  const bf16_t* qg = reinterpret_cast<const bf16_t*>(p.q) + (long)kh * p.dk;
  const bf16_t* kg = reinterpret_cast<const bf16_t*>(p.k) + (long)kh * p.dk;
  const bf16_t* vg = reinterpret_cast<const bf16_t*>(p.v) + (long)h * p.dv;
  const float* pg = p.pre + ((long)row0 * p.H + h) * kPre;
  // A chunk's operands travel into registers two chunks ahead, as raw pieces from clamped places, and are masked as they are staged.
  constexpr int CPR = NP / 8, NQK = (2 * kL * CPR + NT - 1) / NT, NV = (kL * COLS / 4 + NT - 1) / NT, NPR = (kL * kPre / 4 + NT - 1) / NT;
  struct Raw {
    uint4_t qk[NQK];
    bf16_t v[NV][4];
    floatx4 pre[NPR];
  };
  auto fetch = [&](int t0, Raw& r) __attribute__((always_inline)) {
    if (t0 >= len) return;
    const int tl = min(kL, len - t0), ncpr = p.dk / 8;
    if constexpr (VEC) {
#pragma unroll
      for (int x = 0; x < NQK; ++x) {
        const int i = min(tid + NT * x, 2 * kL * CPR - 1), which = i / (kL * CPR), e = i % (kL * CPR);
        const int t = min(e / CPR, tl - 1), c = min(e % CPR, ncpr - 1);
        r.qk[x] = ld16((which ? qg : kg) + (long)(row0 + t0 + t) * (which ? p.qs : p.ks) + c * 8);
      }
    }
#pragma unroll
    for (int x = 0; x < NV; ++x) {
      const int i = min(tid + NT * x, kL * COLS / 4 - 1), t = min(i / (COLS / 4), tl - 1), c = j0 + 4 * (i % (COLS / 4));
      const bf16_t* vr = vg + (long)(row0 + t0 + t) * p.vs;
      if constexpr (VEC) {
        *reinterpret_cast<short4_t*>(r.v[x]) = *reinterpret_cast<const short4_t*>(vr + min(c, p.dv - 4));
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e) r.v[x][e] = vr[min(c + e, p.dv - 1)];
      }
    }
#pragma unroll
    for (int x = 0; x < NPR; ++x) {
      const int i = min(tid + NT * x, kL * kPre / 4 - 1), t = min(i / (kPre / 4), tl - 1), c = i % (kPre / 4);
      r.pre[x] = *reinterpret_cast<const floatx4*>(pg + (long)(t0 + t) * p.H * kPre + 4 * c);
    }
  };
  auto stage = [&](int t0, int buf, const Raw& r) __attribute__((always_inline)) {
    if (t0 >= len) return;
    const int tl = min(kL, len - t0);
    if constexpr (VEC) {
#pragma unroll
      for (int x = 0; x < NQK; ++x) {
        const int i = tid + NT * x;
        if (2 * kL * CPR % NT == 0 || i < 2 * kL * CPR) {
          const int which = i / (kL * CPR), e = i % (kL * CPR), t = e / CPR, c = e % CPR;
          bf16_t* dst = (which ? hq[buf][t] : hk[buf][t]) + 32 * (c >> 2) + 16 * (c & 1) + 4 * ((c >> 1) & 1);
          const uint4_t raw = t >= tl || c >= p.dk / 8 ? uint4_t{0u, 0u, 0u, 0u} : r.qk[x];
          *reinterpret_cast<uint64_t*>(dst) = (uint64_t)raw[1] << 32 | raw[0];
          *reinterpret_cast<uint64_t*>(dst + 8) = (uint64_t)raw[3] << 32 | raw[2];
        }
      }
    } else {
      for (int i = tid; i < 2 * kL * NP; i += NT) {
        const int which = i / (kL * NP), e = i % (kL * NP), t = e / NP, c = e % NP;
        const long row = row0 + t0 + t;
        bf16_t v = 0;
        if (t < tl && c < p.dk) v = which ? qg[row * p.qs + c] : kg[row * p.ks + c];
        (which ? hq[buf][t] : hk[buf][t])[(c & ~31) + 8 * ((c >> 2) & 3) + 4 * ((c >> 4) & 1) + (c & 3)] = v;
      }
    }
#pragma unroll
    for (int x = 0; x < NV; ++x) {
      const int i = tid + NT * x;
      if (kL * COLS / 4 % NT == 0 || i < kL * COLS / 4) {
        const int t = i / (COLS / 4), c = 4 * (i % (COLS / 4));
        floatx4 v;
#pragma unroll
        for (int e = 0; e < 4; ++e) v[e] = t < tl && j0 + c + e < p.dv ? bf2f(r.v[x][e]) : 0.f;
        *reinterpret_cast<floatx4*>(&sv[buf][t][c]) = v;
      }
    }
#pragma unroll
    for (int x = 0; x < NPR; ++x) {
      const int i = tid + NT * x;
      if (kL * kPre / 4 % NT == 0 || i < kL * kPre / 4) {
        const int t = i / (kPre / 4), c = i % (kPre / 4);
        *reinterpret_cast<floatx4*>(&sp[buf][t][4 * c]) = t < tl ? r.pre[x] : floatx4{0.f, 0.f, 0.f, 0.f};
      }
    }
  };
  uint4_t part[NB][3];   // the state's parts as B operands
  auto split = [&]() __attribute__((always_inline)) {
#pragma unroll
    for (int b = 0; b < NB; ++b)
#pragma unroll
      for (int x = 0; x < 4; ++x) {
        float a = S[2 * b + (x >> 1)][2 * (x & 1)], c = S[2 * b + (x >> 1)][2 * (x & 1) + 1];
        part[b][0][x] = upper_halves(a, c);
        a -= cut(a);
        c -= cut(c);
        part[b][1][x] = upper_halves(a, c);
        a -= cut(a);
        c -= cut(c);
        part[b][2][x] = upper_halves(a, c);
      }
  };
  auto mma = [](uint4_t a, uint4_t b, floatx4 c) __attribute__((always_inline)) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(short8, a), __builtin_bit_cast(short8, b), c, 0, 0, 0);
  };
  const int qq = n16 >> 2, pp = n16 & 3;
  auto compute = [&](int t0, int buf) __attribute__((always_inline)) {
    const int tl = min(kL, len - t0);
    // K S and Q S: rows t = 4g + j, column n16 of this wave's tile
    floatx4 y1[3], y2[3];
#pragma unroll
    for (int x = 0; x < 3; ++x) y1[x] = y2[x] = floatx4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int b = 0; b < NB; ++b) {
      const uint4_t kf = ld16(&hk[buf][n16][32 * b + 8 * g]);
#pragma unroll
      for (int x = 0; x < 3; ++x) y1[x] = mma(kf, part[b][x], y1[x]);
    }
#pragma unroll
    for (int b = 0; b < NB; ++b) {
      const uint4_t qf = ld16(&hq[buf][n16][32 * b + 8 * g]);
#pragma unroll
      for (int x = 0; x < 3; ++x) y2[x] = mma(qf, part[b][x], y2[x]);
    }
    float xv[4];
    floatx4 f4[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      f4[j] = *reinterpret_cast<const floatx4*>(&sp[buf][4 * g + j][32]);
      xv[j] = sv[buf][4 * g + j][16 * w + n16] - f4[j][0] * (y1[0][j] + (y1[1][j] + y1[2][j]));
    }
    floatx4 u = {0.f, 0.f, 0.f, 0.f}, o;
    const floatx4 b4 = *reinterpret_cast<const floatx4*>(&sp[buf][n16][4 * g]), p4 = *reinterpret_cast<const floatx4*>(&sp[buf][n16][16 + 4 * g]);
    const float dec = sp[buf][0][35];
#pragma unroll
    for (int j = 0; j < 4; ++j) u = __builtin_amdgcn_mfma_f32_16x16x4f32(b4[j], xv[j], u, 0, 0, 0);
#pragma unroll
    for (int nt = 0; nt < NR; ++nt)
#pragma unroll
      for (int j = 0; j < 4; ++j) S[nt][j] *= dec;
#pragma unroll
    for (int j = 0; j < 4; ++j) o[j] = f4[j][1] * (y2[0][j] + (y2[1][j] + y2[2][j]));
    // state: rows i = 16 nt + 4g + j, column n16
    float us[4], r1[4], r2[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      us[j] = u[j] * f4[j][2];
      r1[j] = us[j] - cut(us[j]);
      r2[j] = r1[j] - cut(r1[j]);
    }
    const uint4_t ub = {upper_halves(us[0], us[1]), upper_halves(us[2], us[3]), upper_halves(r1[0], r1[1]), upper_halves(r1[2], r1[3])};
    const uint4_t ul = {upper_halves(r2[0], r2[1]), upper_halves(r2[2], r2[3]), 0u, 0u};
#pragma unroll
    for (int nt = 0; nt < NR; ++nt) {
      const bf16_t* a0 = &hk[buf][4 * g + qq][32 * (nt >> 1) + 8 * pp + 4 * (nt & 1)];
      const uint64_t kt = __builtin_bit_cast(uint64_t, __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_short4_ptr)(a0)));
      const uint4_t ka = {(unsigned)kt, (unsigned)(kt >> 32), (unsigned)kt, (unsigned)(kt >> 32)};
      S[nt] = mma(ka, ub, S[nt]);
      S[nt] = mma(ka, ul, S[nt]);
    }
#pragma unroll
    for (int j = 0; j < 4; ++j) o = __builtin_amdgcn_mfma_f32_16x16x4f32(p4[j], u[j], o, 0, 0, 0);
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (cv && 4 * g + j < tl) og[(long)(t0 + 4 * g + j) * p.H * p.dv + col] = o[j];
    split();
  };
  Raw ra, rb;
  fetch(0, ra);
  fetch(kL, rb);
  split();
  stage(0, 0, ra);
  fetch(2 * kL, ra);
  __syncthreads();
  for (int t0 = 0; t0 < len; t0 += 2 * kL) {
    compute(t0, 0);
    stage(t0 + kL, 1, rb);
    fetch(t0 + 3 * kL, rb);
    __syncthreads();
    if (t0 + kL >= len) break;
    compute(t0 + kL, 1);
    stage(t0 + 2 * kL, 0, ra);
    fetch(t0 + 4 * kL, ra);
    __syncthreads();
  }
  if (cv) {
#pragma unroll
    for (int nt = 0; nt < NR; ++nt)
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int i = nt * 16 + 4 * g + j;
        if (i < p.dk) Sg[(long)i * p.dv] = S[nt][j];
      }
  }
}

bool al(const void* x, int b) { return reinterpret_cast<uintptr_t>(x) % b == 0; }

template <typename T, int NR>
int launch_step(const HeadDeltaParams& p, int S, hipStream_t st) {
  const dim3 grid((unsigned)S, (unsigned)p.H);
  const bool vec = p.dv % 4 == 0 && al(p.state, 16);
  if (p.dv <= 64) {
    if (vec) head_delta_step_kernel<T, NR, 16, true><<<grid, 256, 0, st>>>(p);
    else head_delta_step_kernel<T, NR, 16, false><<<grid, 256, 0, st>>>(p);
  } else {
    if (vec) head_delta_step_kernel<T, NR, 32, true><<<grid, 512, 0, st>>>(p);
    else head_delta_step_kernel<T, NR, 32, false><<<grid, 512, 0, st>>>(p);
  }
  LK_CHECK_LAUNCH();
  return 0;
}

template <typename T, int NR, int NW>
int launch_chunk(const HeadDeltaParams& p, int S, bool vec, hipStream_t st) {
  const dim3 grid((unsigned)S, (unsigned)p.H, (unsigned)((p.dv + 16 * NW - 1) / (16 * NW)));
  if constexpr (sizeof(T) == 2) {
    constexpr int N2 = NR < 2 ? 2 : NR;
    if (vec) head_delta_chunk_bf16_kernel<N2, NW, true><<<grid, 64 * NW, 0, st>>>(p);
    else head_delta_chunk_bf16_kernel<N2, NW, false><<<grid, 64 * NW, 0, st>>>(p);
  } else {
    if (vec) head_delta_chunk_kernel<T, NR, NW, true><<<grid, 64 * NW, 0, st>>>(p);
    else head_delta_chunk_kernel<T, NR, NW, false><<<grid, 64 * NW, 0, st>>>(p);
  }
  LK_CHECK_LAUNCH();
  return 0;
}

template <typename T, int NR>
int run_nr(const HeadDeltaParams& p, int S, int max_len, hipStream_t st) {
  if (max_len <= 1) return launch_step<T, NR>(p, S, st);
  constexpr int ev = El<T>::V;
  const bool vqk = p.dk % ev == 0 && p.qs % ev == 0 && p.ks % ev == 0 && al(p.q, 16) && al(p.k, 16);
  const int chunks = (max_len + kL - 1) / kL;
  if (S > 65535 || chunks < 1) return -1;
  head_delta_chunk_pre_kernel<T><<<dim3((unsigned)chunks, (unsigned)((p.H + 3) / 4), (unsigned)S), 256, 0, st>>>(p, vqk);
  LK_CHECK_LAUNCH();
  const bool vec = vqk && p.dv % 4 == 0 && p.vs % 4 == 0 && al(p.v, 4 * sizeof(T));
  // workgroups of 64 columns once they fill the chip, of 32 (an operand copy for half as many waves) before that
  return (long)S * p.H * ((p.dv + 63) / 64) >= 512 ? launch_chunk<T, NR, 4>(p, S, vec, st) : launch_chunk<T, NR, 2>(p, S, vec, st);
}

template <typename T>
int run_t(const HeadDeltaParams& p, int S, int max_len, hipStream_t st) {
  if (p.dk <= 16) return run_nr<T, 1>(p, S, max_len, st);
  if (p.dk <= 32) return run_nr<T, 2>(p, S, max_len, st);
  if (p.dk <= 64) return run_nr<T, 4>(p, S, max_len, st);
  if (p.dk <= 128) return run_nr<T, 8>(p, S, max_len, st);
  if (p.dk <= 256) return run_nr<T, 16>(p, S, max_len, st);
  return -1;
}

}  // namespace

int lk_head_delta_pre() { return kPre; }

// T rows of S sequences; max_len 1: single tokens (pre and o unused), else pre [T, H, lk_head_delta_pre()] and o [T, H * dv] f32 scratch
int lk_head_delta(const void* q, long qs, const void* k, long ks, const void* v, long vs, const void* b, long bs, const void* a, long as,
                  const float* dt_bias, const float* A_log, const void* gate, long gs, const float* norm_w, float eps, float* state,
                  const int* cu, const int* slots, const int* positions, int S, long T, int H, int Hk, int dk, int dv, void* out, long os,
                  int max_len, float* pre, float* o, int esz, hipStream_t st) {
  if (S <= 0 || T <= 0) return 0;
  if (H < 1 || Hk < 1 || H % Hk || H > 65535 || dk < 1 || dk > 256 || dv < 1 || dv > 1024 || max_len < 1 || (max_len > 1 && (!pre || !o || !al(pre, 16))))
    return -1;
  HeadDeltaParams p;
  p.q = q; p.k = k; p.v = v; p.b = b; p.a = a; p.gate = gate; p.qs = qs; p.ks = ks; p.vs = vs; p.bs = bs; p.as = as; p.gs = gs;
  p.dt_bias = dt_bias; p.A_log = A_log; p.norm_w = norm_w; p.eps = eps; p.state = state; p.cu = cu; p.slots = slots; p.positions = positions;
  p.H = H; p.Hk = Hk; p.dk = dk; p.dv = dv; p.out = out; p.os = os; p.pre = pre; p.o = o;
  const int rc = esz == 2 ? run_t<bf16_t>(p, S, max_len, st) : run_t<float>(p, S, max_len, st);
  if (rc || max_len <= 1) return rc;
  return lk_head_norm_gate(o, (long)H * dv, gate, gs, esz, norm_w, T, H, dv, eps, 0, out, os, esz, st);
}
