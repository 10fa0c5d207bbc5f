// Per-head products out[t, h, n] = sum_k w[h][n][k] x[t, h * xh + k] (bf16 or f32 rows and weights, f32 accumulation): the
// projections between a head's own space and a latent that all heads share.
//
// Computed transposed (A = weight rows, B = token rows), so a lane ends up with 4 adjacent output columns of one token: one 8- or
// 16-byte store.  grid (token tiles, column tiles, heads); 4 waves as WT x (4 / WT) along tokens x columns, each RT tiles of 16
// tokens x 4 tiles of 16 columns; fragments straight from memory (what the waves of a workgroup share is an L1 hit).
#include "common.h"
#include "kernels.h"
#include "attn_frag.h"

namespace {

template <typename T, int RT, int WT>
__global__ __launch_bounds__(256) void head_linear_kernel(const T* __restrict__ x, long xs, long xh, const T* __restrict__ w, int N, int K,
                                                          long rows, T* __restrict__ out, long os, long oh, int vec, int vst) {
  constexpr int EV = El<T>::V, STEP = 4 * EV, NT = 4, U = RT == 1 ? 4 : 1;
  const int lane = threadIdx.x & 63, wv = threadIdx.x >> 6, n16 = lane & 15, g = lane >> 4;
  const int h = blockIdx.z, c0 = (blockIdx.y * (4 / WT) + wv / WT) * 16 * NT;
  const long t0 = ((long)blockIdx.x * WT + wv % WT) * 16 * RT;
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
  int kb = 0;
  if (vec) {
    for (; kb + U * STEP <= K; kb += U * STEP) {
      uint4_t a[U][NT], b[U][RT];
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const int k = kb + (4 * u + g) * EV;
#pragma unroll
        for (int c = 0; c < NT; ++c) a[u][c] = ld16(wr[c] + k);
#pragma unroll
        for (int r = 0; r < RT; ++r) b[u][r] = ld16(xr[r] + k);
      }
#pragma unroll
      for (int u = 0; u < U; ++u)
#pragma unroll
        for (int r = 0; r < RT; ++r)
#pragma unroll
          for (int c = 0; c < NT; ++c) acc[r][c] = mma_qk<T>(a[u][c], b[u][r], acc[r][c]);
    }
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
    for (int c = 0; c < NT; ++c) {
      const int n = c0 + 16 * c + 4 * g;
      if (vst && n + 4 <= N) {
        if constexpr (sizeof(T) == 2) {
          short4_t v;
#pragma unroll
          for (int j = 0; j < 4; ++j) v[j] = (short)f2bf(acc[r][c][j]);
          *reinterpret_cast<short4_t*>(orow + n) = v;
        } else {
          *reinterpret_cast<floatx4*>(orow + n) = acc[r][c];
        }
      } else {
#pragma unroll
        for (int j = 0; j < 4; ++j)
          if (n + j < N) El<T>::st(orow + n + j, acc[r][c][j]);
      }
    }
  }
}

template <typename T>
int head_linear_t(const void* x, long xs, long xh, const void* w, int H, int N, int K, long rows, void* out, long os, long oh, int vec, int vst,
                  hipStream_t st) {
#define LK_HEAD(RT, WT)                                                                                                                     \
  head_linear_kernel<T, RT, WT><<<dim3((unsigned)((rows + 16 * RT * WT - 1) / (16 * RT * WT)), (unsigned)((N + 64 * (4 / WT) - 1) / (64 * (4 / WT))), \
                                       (unsigned)H), 256, 0, st>>>((const T*)x, xs, xh, (const T*)w, N, K, rows, (T*)out, os, oh, vec, vst)
  if (rows > 128) LK_HEAD(4, 2);
  else LK_HEAD(1, 4);
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
