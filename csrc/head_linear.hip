// Per-head products out[t, h, n] = sum_k w[h][n][k] x[t, h * xh + k] (bf16 or f32 rows and weights, f32 accumulation): the
// projections between a head's own space and a latent that all heads share.
//
// Computed transposed (A = weight rows, B = token rows), so a lane ends up with 4 adjacent output columns of one token: one 8- or
// 16-byte store.  Grids run over the heads fastest: rows lie a power of two apart, and neighbours that differ in the head spread over
// the memory channels and keep each XCD on a few heads' weights.
//
// Many rows: a workgroup owns 128 tokens x 128 columns of a head, its 4 waves 64 x 64 quarters; both operands of a 128-byte step of
// the contraction are fetched once per workgroup (the next step's under this step's products) and staged in LDS, rows padded to
// 144 bytes.  Few rows, and sizes the vector loads do not divide: fragments straight from memory, a wave owns 16 tokens x 64 columns.
#include "common.h"
#include "kernels.h"
#include "attn_frag.h"

namespace {

// the 4 adjacent columns n .. n + 3 of a token's row
template <typename T>
LK_DEVICE void store4(T* row, int n, int N, int vst, const floatx4& v) {
  if (vst && n + 4 <= N) {
    if constexpr (sizeof(T) == 2) {
      short4_t b;
#pragma unroll
      for (int j = 0; j < 4; ++j) b[j] = (short)f2bf(v[j]);
      *reinterpret_cast<short4_t*>(row + n) = b;
    } else {
      *reinterpret_cast<floatx4*>(row + n) = v;
    }
  } else {
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (n + j < N) El<T>::st(row + n + j, v[j]);
  }
}

template <typename T>
__global__ __launch_bounds__(256) void head_linear_lds_kernel(const T* __restrict__ x, long xs, long xh, const T* __restrict__ w, int N, int K,
                                                              long rows, T* __restrict__ out, long os, long oh, int vst) {
  constexpr int EV = El<T>::V, KS = 8 * EV, TM = 128, TN = 128;
  __shared__ uint4_t sx[2][TM][9];
  __shared__ uint4_t sw[2][TN][9];
  const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6, n16 = lane & 15, g = lane >> 4;
  const int h = blockIdx.x, c0 = blockIdx.y * TN;
  const long t0 = (long)blockIdx.z * TM;
  const int pr = tid >> 3, ps = tid & 7;   // this thread's pieces: rows pr + 32 i, segment ps
  const T* xp[4];
  const T* wp[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) {   // rows behind the end read a valid row whose results are not stored
    xp[i] = x + min(t0 + pr + 32 * i, rows - 1) * xs + h * xh;
    wp[i] = w + ((long)h * N + min(c0 + pr + 32 * i, N - 1)) * K;
  }
  uint4_t rx[4], rw[4];
  auto fetch = [&](int kb) {
    const int k = kb + ps * EV;
    const bool in = k < K;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      rx[i] = ld16(xp[i] + (in ? k : 0));
      rw[i] = ld16(wp[i] + (in ? k : 0));
    }
  };
  auto stage = [&](int buf, int kb) {
    const bool in = kb + ps * EV < K;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      sx[buf][pr + 32 * i][ps] = in ? rx[i] : uint4_t{0u, 0u, 0u, 0u};
      sw[buf][pr + 32 * i][ps] = in ? rw[i] : uint4_t{0u, 0u, 0u, 0u};
    }
  };
  const int wt = wv >> 1, wc = wv & 1;
  floatx4 acc[4][4];
#pragma unroll
  for (int r = 0; r < 4; ++r)
#pragma unroll
    for (int c = 0; c < 4; ++c) acc[r][c] = floatx4{0.f, 0.f, 0.f, 0.f};
  fetch(0);
  stage(0, 0);
  __syncthreads();
  int cur = 0;
  for (int kb = 0; kb < K; kb += KS) {
    const bool more = kb + KS < K;
    if (more) fetch(kb + KS);
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      uint4_t a[4], b[4];
#pragma unroll
      for (int c = 0; c < 4; ++c) a[c] = sw[cur][64 * wc + 16 * c + n16][4 * u + g];
#pragma unroll
      for (int r = 0; r < 4; ++r) b[r] = sx[cur][64 * wt + 16 * r + n16][4 * u + g];
#pragma unroll
      for (int r = 0; r < 4; ++r)
#pragma unroll
        for (int c = 0; c < 4; ++c) acc[r][c] = mma_qk<T>(a[c], b[r], acc[r][c]);
    }
    if (more) stage(cur ^ 1, kb + KS);
    __syncthreads();
    cur ^= 1;
  }
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const long t = t0 + 64 * wt + 16 * r + n16;
    if (t >= rows) continue;
#pragma unroll
    for (int c = 0; c < 4; ++c) store4<T>(out + t * os + h * oh, c0 + 64 * wc + 16 * c + 4 * g, N, vst, acc[r][c]);
  }
}

template <typename T, int RT, int WT>
__global__ __launch_bounds__(256) void head_linear_kernel(const T* __restrict__ x, long xs, long xh, const T* __restrict__ w, int N, int K,
                                                          long rows, T* __restrict__ out, long os, long oh, int vec, int vst) {
  constexpr int EV = El<T>::V, STEP = 4 * EV, NT = 4, U = 2;
  const int lane = threadIdx.x & 63, wv = threadIdx.x >> 6, n16 = lane & 15, g = lane >> 4;
  const int h = blockIdx.x, c0 = (blockIdx.y * (4 / WT) + wv / WT) * 16 * NT;
  const long t0 = ((long)blockIdx.z * WT + wv % WT) * 16 * RT;
  if (t0 >= rows || c0 >= N) return;   // no barrier in this kernel
  const T* xr[RT];
#pragma unroll
  for (int r = 0; r < RT; ++r) xr[r] = x + min(t0 + 16 * r + n16, rows - 1) * xs + h * xh;
  const T* wr[NT];
#pragma unroll
  for (int c = 0; c < NT; ++c) wr[c] = w + ((long)h * N + min(c0 + 16 * c + n16, N - 1)) * K;
  floatx4 acc[RT][NT];
#pragma unroll
  for (int r = 0; r < RT; ++r)
#pragma unroll
    for (int c = 0; c < NT; ++c) acc[r][c] = floatx4{0.f, 0.f, 0.f, 0.f};
  // whole steps as plain vector loads, U of them requested together, the next group's ahead of this group's products
  int kb = 0;
  const int groups = vec ? K / (U * STEP) : 0;
  if (groups > 0) {
    uint4_t a[2][U][NT], b[2][U][RT];
    auto load = [&](int p, int k0) {
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const int k = k0 + (4 * u + g) * EV;
#pragma unroll
        for (int c = 0; c < NT; ++c) a[p][u][c] = ld16(wr[c] + k);
#pragma unroll
        for (int r = 0; r < RT; ++r) b[p][u][r] = ld16(xr[r] + k);
      }
    };
    auto mul = [&](int p) {
#pragma unroll
      for (int u = 0; u < U; ++u)
#pragma unroll
        for (int r = 0; r < RT; ++r)
#pragma unroll
          for (int c = 0; c < NT; ++c) acc[r][c] = mma_qk<T>(a[p][u][c], b[p][u][r], acc[r][c]);
    };
    load(0, 0);
    for (int i = 0; i < groups; i += 2) {
      if (i + 1 < groups) load(1, (i + 1) * U * STEP);
      mul(0);
      if (i + 1 < groups) {
        if (i + 2 < groups) load(0, (i + 2) * U * STEP);
        mul(1);
      }
    }
    kb = groups * U * STEP;
  }
  for (; kb < K; kb += STEP) {
    const int k = kb + g * EV;
    uint4_t a[NT], b[RT];
#pragma unroll
    for (int c = 0; c < NT; ++c) a[c] = frag<T>(wr[c], k, K, vec);
#pragma unroll
    for (int r = 0; r < RT; ++r) b[r] = frag<T>(xr[r], k, K, vec);
#pragma unroll
    for (int r = 0; r < RT; ++r)
#pragma unroll
      for (int c = 0; c < NT; ++c) acc[r][c] = mma_qk<T>(a[c], b[r], acc[r][c]);
  }
  // accumulator j of this lane: output column 16 c + 4 g + j of token 16 r + n16
#pragma unroll
  for (int r = 0; r < RT; ++r) {
    const long t = t0 + 16 * r + n16;
    if (t >= rows) continue;
    T* orow = out + t * os + h * oh;
#pragma unroll
    for (int c = 0; c < NT; ++c) store4<T>(orow, c0 + 16 * c + 4 * g, N, vst, acc[r][c]);
  }
}

template <typename T>
int head_linear_t(const void* x, long xs, long xh, const void* w, int H, int N, int K, long rows, void* out, long os, long oh, int vec, int vst,
                  hipStream_t st) {
  if (rows > 65535L * 64) return -1;
#define LK_HEAD(RT, WT)                                                                                                                      \
  head_linear_kernel<T, RT, WT><<<dim3((unsigned)H, (unsigned)((N + 64 * (4 / WT) - 1) / (64 * (4 / WT))),                                   \
                                       (unsigned)((rows + 16 * RT * WT - 1) / (16 * RT * WT))), 256, 0, st>>>(                              \
      (const T*)x, xs, xh, (const T*)w, N, K, rows, (T*)out, os, oh, vec, vst)
  if (rows > 128 && vec)
    head_linear_lds_kernel<T><<<dim3((unsigned)H, (unsigned)((N + 127) / 128), (unsigned)((rows + 127) / 128)), 256, 0, st>>>(
        (const T*)x, xs, xh, (const T*)w, N, K, rows, (T*)out, os, oh, vst);
  else
    LK_HEAD(1, 4);
#undef LK_HEAD
  LK_CHECK_LAUNCH();
  return 0;
}

}  // namespace

int lk_head_linear(const void* x, long xs, long xh, const void* w, int H, int N, int K, long rows, void* out, long os, long oh, int esz,
                   hipStream_t st) {
  if (rows <= 0) return 0;
  if (H < 1 || H > 65535 || N < 1 || K < 1 || (N + 63) / 64 > 65535) return -1;
  const int ev = 16 / esz;
  const auto a16 = [](const void* p, int b) { return reinterpret_cast<uintptr_t>(p) % b == 0; };
  const int vec = K % ev == 0 && xs % ev == 0 && xh % ev == 0 && a16(x, 16) && a16(w, 16);
  const int vst = os % 4 == 0 && oh % 4 == 0 && a16(out, 4 * esz);
  return esz == 2 ? head_linear_t<bf16_t>(x, xs, xh, w, H, N, K, rows, out, os, oh, vec, vst, st)
                  : head_linear_t<float>(x, xs, xh, w, H, N, K, rows, out, os, oh, vec, vst, st);
}
