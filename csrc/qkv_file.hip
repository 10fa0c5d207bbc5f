// Queries, keys and values of one step from a fused projection [q: H dim | k: G dim | v: G vdim] (bf16 or f32 rows) to where attention
// reads them, all of it in f32: the projection's bias, an optional RMS norm over ALL q rows and over all k rows of the projection
// (before it is split into heads) with a weight per row, the rotation of adjacent pairs (2 i, 2 i + 1) of a head's first `rot`
// dimensions by position * freq[i] (cos and sin times `mag`).  q is rewritten in place; k goes to the paged cache
// [blocks, G, BS, dim], v to the key-contiguous one [blocks, G, vdim, BS], at slots[t] (< 0: nothing is cached).
//
// One workgroup per token.  A thread holds 16-byte pieces of the row (a pair never straddles two pieces: heads are multiples of a
// piece), so the row is read once and everything between load and store is in registers.  With many rows the values are filed by a kernel
// of their own: 16 tokens x 64 columns turn round in LDS, so that a column's run of tokens is written in 16-byte pieces.
#include "common.h"
#include "kernels.h"
#include "attn_frag.h"

namespace {

constexpr int kMaxRot = 256;

struct FileParams {
  void* u;
  long us;
  int H, G, dim, vdim, BS;
  const float* bias;   // [H dim + G dim + G vdim] or null
  const float* qw;     // [H dim], [G dim] or both null (no norm)
  const float* kw;
  float inv_nq, inv_nk, eps;
  int rot;
  const float* freq;
  float mag;
  const int* positions;
  void* kc;
  void* vc;
  const int* slots;
  int v_apart;         // the values are filed by file_values_kernel
};

template <typename T, int MAXC>
__global__ __launch_bounds__(256) void qkv_file_kernel(FileParams p) {
  constexpr int EV = El<T>::V;
  __shared__ float scs[kMaxRot / 2], ssn[kMaxRot / 2], red[4];
  const long t = blockIdx.x;
  const int tid = threadIdx.x, slot = p.slots[t];
  const int nq = p.H * p.dim, nk = p.G * p.dim, n = nq + nk + (p.v_apart ? 0 : p.G * p.vdim);
  T* row = reinterpret_cast<T*>(p.u) + t * p.us;
  for (int i = tid; i < p.rot / 2; i += 256) {
    float sn, cs;
    sincosf((float)p.positions[t] * p.freq[i], &sn, &cs);
    scs[i] = cs * p.mag;
    ssn[i] = sn * p.mag;
  }
  float x[MAXC][EV];
  float sq = 0.f, sk = 0.f;
#pragma unroll
  for (int i = 0; i < MAXC; ++i) {
    const int c = (tid + 256 * i) * EV;
    if (c < n) {
      const uint4_t raw = ld16(row + c);
      const T* e = reinterpret_cast<const T*>(&raw);
#pragma unroll
      for (int j = 0; j < EV; ++j) x[i][j] = El<T>::ld(e + j);
      if (p.bias) {
#pragma unroll
        for (int j = 0; j < EV; j += 4) {
          const floatx4 b = *reinterpret_cast<const floatx4*>(p.bias + c + j);
#pragma unroll
          for (int k = 0; k < 4; ++k) x[i][j + k] += b[k];
        }
      }
      float s = 0.f;
#pragma unroll
      for (int j = 0; j < EV; ++j) s += x[i][j] * x[i][j];
      if (c < nq) sq += s;
      else if (c < nq + nk) sk += s;
    }
  }
  float iq = 1.f, ik = 1.f;
  if (p.qw) {
    iq = 1.f / sqrtf(block_sum<4>(sq, red) * p.inv_nq + p.eps);
    ik = 1.f / sqrtf(block_sum<4>(sk, red) * p.inv_nk + p.eps);
  }
  __syncthreads();
  const long blk = slot >= 0 ? slot / p.BS : 0;
  const int off = slot >= 0 ? slot % p.BS : 0;
#pragma unroll
  for (int i = 0; i < MAXC; ++i) {
    const int c = (tid + 256 * i) * EV;
    if (c >= n || (slot < 0 && c >= nq)) continue;
    if (c >= nq + nk) {
      const int vc = c - nq - nk, gh = vc / p.vdim, d = vc % p.vdim;
      T* dst = reinterpret_cast<T*>(p.vc) + ((blk * p.G + gh) * p.vdim + d) * (long)p.BS + off;
#pragma unroll
      for (int j = 0; j < EV; ++j) El<T>::st(dst + (long)j * p.BS, x[i][j]);
      continue;
    }
    const bool isq = c < nq;
    const int cc = isq ? c : c - nq, hd = cc / p.dim, d = cc % p.dim;
    float y[EV];
#pragma unroll
    for (int j = 0; j < EV; ++j) y[j] = x[i][j];
    if (p.qw) {
      const float inv = isq ? iq : ik;
      const float* w = (isq ? p.qw : p.kw) + cc;
#pragma unroll
      for (int j = 0; j < EV; ++j) y[j] *= inv * w[j];
    }
    if (d < p.rot) {
#pragma unroll
      for (int j = 0; j < EV; j += 2) {
        if (d + j < p.rot) {
          const float cs = scs[(d + j) / 2], sn = ssn[(d + j) / 2], a = y[j], b = y[j + 1];
          y[j] = rot_lo(a, b, cs, sn);
          y[j + 1] = rot_hi(a, b, cs, sn);
        }
      }
    }
    alignas(16) T o[EV];
#pragma unroll
    for (int j = 0; j < EV; ++j) El<T>::st(o + j, y[j]);
    T* dst = isq ? row + c : reinterpret_cast<T*>(p.kc) + ((blk * p.G + hd) * p.BS + off) * (long)p.dim + d;
    *reinterpret_cast<uint4_t*>(dst) = *reinterpret_cast<const uint4_t*>(o);
  }
}

// grid (16 tokens, 64 value columns), 128 threads
constexpr int kVTok = 16, kVCol = 64;
template <typename T>
__global__ __launch_bounds__(128) void file_values_kernel(FileParams p, long rows) {
  constexpr int EV = El<T>::V;
  __shared__ __attribute__((aligned(16))) T sv[kVCol][kVTok + EV];
  const int tid = threadIdx.x, nv = p.G * p.vdim, c0 = blockIdx.y * kVCol, v0 = (p.H + p.G) * p.dim;
  const long t0 = (long)blockIdx.x * kVTok;
  const int tl = (int)min((long)kVTok, rows - t0);
  for (int i = tid; i < kVTok * kVCol / EV; i += 128) {
    const int t = i / (kVCol / EV), c = (i % (kVCol / EV)) * EV;
    if (t < tl && c0 + c < nv) {   // (nv is a multiple of a piece)
      const uint4_t raw = ld16(reinterpret_cast<const T*>(p.u) + (t0 + t) * p.us + v0 + c0 + c);
      const T* e = reinterpret_cast<const T*>(&raw);
#pragma unroll
      for (int j = 0; j < EV; ++j) {
        if (p.bias) El<T>::st(&sv[c + j][t], El<T>::ld(e + j) + p.bias[v0 + c0 + c + j]);
        else sv[c + j][t] = e[j];
      }
    }
  }
  __syncthreads();
  for (int i = tid; i < kVCol * kVTok / EV; i += 128) {
    const int c = i / (kVTok / EV), tb = (i % (kVTok / EV)) * EV;
    if (c0 + c >= nv || tb >= tl) continue;
    const int gh = (c0 + c) / p.vdim, d = (c0 + c) % p.vdim, n = min(EV, tl - tb), s0 = p.slots[t0 + tb];
    auto place = [&](int slot) { return reinterpret_cast<T*>(p.vc) + (((long)(slot / p.BS) * p.G + gh) * p.vdim + d) * p.BS + slot % p.BS; };
    bool run = n == EV && s0 >= 0 && s0 % EV == 0;
    for (int j = 1; j < n; ++j) run = run && p.slots[t0 + tb + j] == s0 + j;
    if (run) {
      *reinterpret_cast<uint4_t*>(place(s0)) = *reinterpret_cast<const uint4_t*>(&sv[c][tb]);
    } else {
      for (int j = 0; j < n; ++j) {
        const int slot = p.slots[t0 + tb + j];
        if (slot >= 0) *place(slot) = sv[c][tb + j];
      }
    }
  }
}

template <typename T>
int launch_file(FileParams p, long T_, hipStream_t st) {
  p.v_apart = T_ >= 256 && p.BS % El<T>::V == 0 && (reinterpret_cast<uintptr_t>(p.vc) & 15) == 0;
  if (p.v_apart) {
    file_values_kernel<T><<<dim3((unsigned)((T_ + kVTok - 1) / kVTok), (unsigned)((p.G * p.vdim + kVCol - 1) / kVCol)), 128, 0, st>>>(p, T_);
    LK_CHECK_LAUNCH();
  }
  const int n = (p.H + p.G) * p.dim + (p.v_apart ? 0 : p.G * p.vdim), per = 256 * El<T>::V;
  const unsigned g = (unsigned)T_;
  if (n <= per) qkv_file_kernel<T, 1><<<g, 256, 0, st>>>(p);
  else if (n <= 2 * per) qkv_file_kernel<T, 2><<<g, 256, 0, st>>>(p);
  else if (n <= 4 * per) qkv_file_kernel<T, 4><<<g, 256, 0, st>>>(p);
  else if (n <= 8 * per) qkv_file_kernel<T, 8><<<g, 256, 0, st>>>(p);
  else if (n <= 16 * per) qkv_file_kernel<T, 16><<<g, 256, 0, st>>>(p);
  else return -1;
  LK_CHECK_LAUNCH();
  return 0;
}

}  // namespace

int lk_qkv_file(void* u, long us, long T, int H, int G, int dim, int vdim, const float* bias, const float* qw, const float* kw, int norm_q,
                int norm_k, float eps, int rot, const float* freq, float mag, const int* positions, void* kc, void* vc, const int* slots,
                int BS, int esz, hipStream_t st) {
  if (T <= 0) return 0;
  const int ev = 16 / esz;
  if (H < 1 || G < 1 || dim < 1 || vdim < 1 || dim % ev || vdim % ev || BS < 1 || us % ev || reinterpret_cast<uintptr_t>(u) % 16 ||
      reinterpret_cast<uintptr_t>(kc) % 16 || reinterpret_cast<uintptr_t>(bias) % 16 || rot < 0 || rot % 2 || rot > dim || rot > kMaxRot ||
      (rot > 0 && !freq) || (qw == nullptr) != (kw == nullptr) || (qw && (norm_q < 1 || norm_k < 1)))
    return -1;
  FileParams p;
  p.u = u; p.us = us; p.H = H; p.G = G; p.dim = dim; p.vdim = vdim; p.BS = BS; p.bias = bias; p.qw = qw; p.kw = kw;
  p.inv_nq = qw ? 1.f / (float)norm_q : 0.f; p.inv_nk = qw ? 1.f / (float)norm_k : 0.f;
  p.eps = eps; p.rot = rot; p.freq = freq; p.mag = mag; p.positions = positions; p.kc = kc; p.vc = vc; p.slots = slots; p.v_apart = 0;
  return esz == 2 ? launch_file<bf16_t>(p, T, st) : launch_file<float>(p, T, st);
}
