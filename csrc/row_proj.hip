// Skinny projections of normed rows whose results stay f32 (h bf16 or f32, weights in the same type, MFMA products summed in
// f32), with what follows them in the same kernel:
//
//   lk_gate_proj      z = W h + b,  c = cap tanh(z / cap);  columns [0, H): c (log input gates), [H, 2H): log sigmoid(c) (log
//                     forget gates)
//   lk_router_choice  z = W h;  scores s = softmax(z) or sigmoid(z) (evaluated in f64);  choice scores c = s + correction;
//                     experts in equal groups of neighbours, a group's score = the largest c in it or the sum of its two
//                     largest; only the `keep` best groups can be chosen; the `top` largest c among those; weights
//                     s / (sum of the chosen s + 1e-20) * scale
//
// A workgroup owns 16 rows; its 8 waves split the contraction (each wave's fragments come straight from memory: the rows are
// few and the weights are read once per 16 rows), partial tiles are summed through LDS in wave order.
#include "common.h"
#include "kernels.h"
#include "attn_frag.h"

namespace {

constexpr int kWaves = 8;
constexpr int kRowTile = 16;
constexpr int kCols = 64;            // weight rows per round
constexpr int kMaxExperts = 1024;
constexpr int kMaxTop = 64;

// zs[16][ldz] = the f32 products of this workgroup's rows with the N weight rows
template <typename T>
LK_DEVICE void project(const T* __restrict__ h, long hs, const T* __restrict__ w, int N, int K, long rows, int vec, float* red, float* zs,
                       int ldz) {
  constexpr int EV = El<T>::V, STEP = 4 * EV, NT = kCols / 16, U = 4;
  const int lane = threadIdx.x & 63, wv = threadIdx.x >> 6, n16 = lane & 15, g = lane >> 4;
  const long t0 = (long)blockIdx.x * kRowTile;
  const T* hr = h + min(t0 + n16, rows - 1) * hs;
  const int steps = (K + STEP - 1) / STEP, per = (steps + kWaves - 1) / kWaves;
  const int k0 = wv * per * STEP, k1 = min(K, (wv + 1) * per * STEP);
  for (int c0 = 0; c0 < N; c0 += kCols) {
    const T* wr[NT];
#pragma unroll
    for (int c = 0; c < NT; ++c) wr[c] = w + (long)min(c0 + 16 * c + n16, N - 1) * K;
    floatx4 acc[NT];
#pragma unroll
    for (int c = 0; c < NT; ++c) acc[c] = floatx4{0.f, 0.f, 0.f, 0.f};
    const int nt = min(NT, (N - c0 + 15) / 16);
    int kb = k0;
    if (vec) {
      for (; kb + U * STEP <= k1; kb += U * STEP) {   // U whole steps: loads requested together ahead of their products
        uint4_t a[U], b[U][NT];
#pragma unroll
        for (int x = 0; x < U; ++x) {
          const int k = kb + (4 * x + g) * EV;
          a[x] = ld16(hr + k);
#pragma unroll
          for (int c = 0; c < NT; ++c)
            if (c < nt) b[x][c] = ld16(wr[c] + k);
        }
#pragma unroll
        for (int x = 0; x < U; ++x)
#pragma unroll
          for (int c = 0; c < NT; ++c)
            if (c < nt) acc[c] = mma_qk<T>(a[x], b[x][c], acc[c]);
      }
    }
    for (; kb < k1; kb += STEP) {
      const int k = kb + g * EV;
      const uint4_t a = frag<T>(hr, k, K, vec);
#pragma unroll
      for (int c = 0; c < NT; ++c)
        if (c < nt) acc[c] = mma_qk<T>(a, frag<T>(wr[c], k, K, vec), acc[c]);
    }
    // accumulator j of this lane: row 4 g + j, column 16 c + n16
    __syncthreads();   // the previous round's sums have been read
#pragma unroll
    for (int c = 0; c < NT; ++c)
#pragma unroll
      for (int j = 0; j < 4; ++j) red[(wv * kRowTile + 4 * g + j) * kCols + 16 * c + n16] = acc[c][j];
    __syncthreads();
    for (int i = threadIdx.x; i < kRowTile * kCols; i += kWaves * 64) {
      const int r = i / kCols, c = i % kCols;
      if (c0 + c < N) {
        float s = 0.f;
#pragma unroll
        for (int x = 0; x < kWaves; ++x) s += red[(x * kRowTile + r) * kCols + c];
        zs[r * ldz + c0 + c] = s;
      }
    }
  }
  __syncthreads();
}

template <typename T>
__global__ __launch_bounds__(kWaves * 64) void gate_proj_kernel(const T* __restrict__ h, long hs, const T* __restrict__ w,
                                                                const float* __restrict__ bias, int N, int K, long rows, float cap,
                                                                int vec, float* __restrict__ out) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  float* red = lds;
  float* zs = lds + kWaves * kRowTile * kCols;
  project<T>(h, hs, w, N, K, rows, vec, red, zs, N);
  const long t0 = (long)blockIdx.x * kRowTile;
  for (int i = threadIdx.x; i < kRowTile * N; i += kWaves * 64) {
    const int r = i / N, c = i % N;
    if (t0 + r < rows) {
      float v = cap * tanhf((zs[i] + bias[c]) / cap);
      if (2 * c >= N) v = v >= 0.f ? -log1pf(expf(-v)) : v - log1pf(expf(v));
      out[(t0 + r) * N + c] = v;
    }
  }
}

// the lanes' pair with the larger value, the smaller index on equal values
LK_DEVICE void wave_argmax(double& s, int& i) {
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) {
    const double so = __shfl_xor(s, o, 64);
    const int io = __shfl_xor(i, o, 64);
    if (so > s || (so == s && io < i)) {
      s = so;
      i = io;
    }
  }
}

LK_DEVICE double wave_sum_d(double v) {
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) v += __shfl_xor(v, o, 64);
  return v;
}

// EPL: choice scores per lane (experts lane, lane + 64, ...)
template <typename T, int EPL>
__global__ __launch_bounds__(kWaves * 64) void router_choice_kernel(const T* __restrict__ h, long hs, const T* __restrict__ w, int E, int K,
                                                                    long rows, int top, int groups, int keep, float scale, int score,
                                                                    const float* __restrict__ corr, int gscore, int vec,
                                                                    int* __restrict__ experts, float* __restrict__ weights) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  float* red = lds;
  float* zs = lds + max(kWaves * kRowTile * kCols, 2 * kWaves * E);
  project<T>(h, hs, w, E, K, rows, vec, red, zs, E);
  double* sc = reinterpret_cast<double*>(lds) + (long)(threadIdx.x >> 6) * E;   // this wave's scores: the partial sums have been consumed
  const int lane = threadIdx.x & 63, wv = threadIdx.x >> 6, per = E / groups;
  const double ninf = -__builtin_huge_val();
  for (int r = wv; r < kRowTile; r += kWaves) {
    const long t = (long)blockIdx.x * kRowTile + r;
    if (t >= rows) break;
    const float* z = zs + r * E;
    float zm = -__builtin_huge_valf();
    for (int e = lane; e < E; e += 64) zm = fmaxf(zm, z[e]);
    zm = wave_max(zm);
    // every lane evaluates its experts' scores once; LDS publishes them to the group scores and the choice
    double c[EPL], den = 0.0;
#pragma unroll
    for (int i = 0; i < EPL; ++i) {
      const int e = lane + 64 * i;
      c[i] = e < E ? (score == 1 ? exp((double)z[e] - (double)zm) : 1.0 / (1.0 + exp(-(double)z[e]))) : 0.0;
      den += c[i];
    }
    const double inv = score == 1 ? 1.0 / wave_sum_d(den) : 1.0;
#pragma unroll
    for (int i = 0; i < EPL; ++i) {
      const int e = lane + 64 * i;
      if (e < E) {
        c[i] *= inv;
        sc[e] = c[i];
        c[i] += corr ? (double)corr[e] : 0.0;
      } else {
        c[i] = ninf;
      }
    }
    __builtin_amdgcn_wave_barrier();
    if (groups > 1) {   // at most 64 groups (host check): lane x holds group x's score
      double mine = ninf;
      if (lane < groups) {
        double b1 = ninf, b2 = ninf;
        for (int j = 0; j < per; ++j) {
          const int e = lane * per + j;
          const double v = sc[e] + (corr ? (double)corr[e] : 0.0);
          if (v > b1) { b2 = b1; b1 = v; } else if (v > b2) { b2 = v; }
        }
        mine = gscore == 1 ? b1 : b1 + (per > 1 ? b2 : 0.0);
      }
      bool kept = false;
      for (int k = 0; k < keep; ++k) {
        double bs = kept ? ninf : mine;
        int bi = kept || lane >= groups ? 64 + lane : lane;
        wave_argmax(bs, bi);
        if (bi == lane) kept = true;
      }
      const unsigned long long mask = __ballot(kept);
#pragma unroll
      for (int i = 0; i < EPL; ++i) {
        const int e = lane + 64 * i;
        if (e < E && !((mask >> (e / per)) & 1ull)) c[i] = ninf;
      }
    }
    double chosen_s = 0.0, sum = 0.0;   // lane k holds the k-th choice
    int chosen_e = 0;
    for (int k = 0; k < top; ++k) {
      double bs = ninf;
      int bi = 0x7fffffff;
#pragma unroll
      for (int i = 0; i < EPL; ++i)
        if (c[i] > bs) { bs = c[i]; bi = lane + 64 * i; }
      wave_argmax(bs, bi);
      if (bi >= E) bi = 0;              // nothing left to choose (NaN scores): keep the indices in range
#pragma unroll
      for (int i = 0; i < EPL; ++i)
        if (bi == lane + 64 * i) c[i] = ninf;
      const double s = sc[bi];
      if (lane == k) { chosen_s = s; chosen_e = bi; }
      sum += s;
    }
    if (lane < top) {
      experts[t * top + lane] = chosen_e;
      weights[t * top + lane] = (float)(chosen_s / (sum + 1e-20) * (double)scale);
    }
  }
}

int vec_ok(const void* h, long hs, const void* w, int K, int esz) {
  const int ev = 16 / esz;
  return K % ev == 0 && hs % ev == 0 && reinterpret_cast<uintptr_t>(h) % 16 == 0 && reinterpret_cast<uintptr_t>(w) % 16 == 0;
}

template <typename T>
int gate_t(const void* h, long hs, const void* w, const float* bias, int N, int K, long rows, float cap, int vec, float* out, hipStream_t st) {
  const size_t lds = sizeof(float) * (kWaves * kRowTile * kCols + (size_t)kRowTile * N);
  if (lds > 128 * 1024) return -1;
  LK_SET_MAX_LDS(gate_proj_kernel<T>, 128 * 1024);
  gate_proj_kernel<T><<<(unsigned)((rows + kRowTile - 1) / kRowTile), kWaves * 64, lds, st>>>((const T*)h, hs, (const T*)w, bias, N, K, rows, cap,
                                                                                             vec, out);
  LK_CHECK_LAUNCH();
  return 0;
}

template <typename T, int EPL>
int router_e(const void* h, long hs, const void* w, int E, int K, long rows, int top, int groups, int keep, float scale, int score,
             const float* corr, int gscore, int vec, int* experts, float* weights, hipStream_t st) {
  const size_t lds = sizeof(float) * ((size_t)(kWaves * kRowTile * kCols > 2 * kWaves * E ? kWaves * kRowTile * kCols : 2 * kWaves * E) +
                                      (size_t)kRowTile * E);
  if (lds > 128 * 1024) return -1;
  LK_SET_MAX_LDS((router_choice_kernel<T, EPL>), 128 * 1024);
  router_choice_kernel<T, EPL><<<(unsigned)((rows + kRowTile - 1) / kRowTile), kWaves * 64, lds, st>>>(
      (const T*)h, hs, (const T*)w, E, K, rows, top, groups, keep, scale, score, corr, gscore, vec, experts, weights);
  LK_CHECK_LAUNCH();
  return 0;
}

template <typename T>
int router_t(const void* h, long hs, const void* w, int E, int K, long rows, int top, int groups, int keep, float scale, int score,
             const float* corr, int gscore, int vec, int* experts, float* weights, hipStream_t st) {
  if (E <= 64) return router_e<T, 1>(h, hs, w, E, K, rows, top, groups, keep, scale, score, corr, gscore, vec, experts, weights, st);
  if (E <= 256) return router_e<T, 4>(h, hs, w, E, K, rows, top, groups, keep, scale, score, corr, gscore, vec, experts, weights, st);
  return router_e<T, 16>(h, hs, w, E, K, rows, top, groups, keep, scale, score, corr, gscore, vec, experts, weights, st);
}

}  // namespace

int lk_gate_proj(const void* h, long hs, const void* w, const float* bias, int N, int K, long rows, float cap, float* out, int esz,
                 hipStream_t st) {
  if (rows <= 0) return 0;
  if (N < 2 || N % 2 || K < 1 || !(cap > 0.f) || !bias) return -1;
  const int vec = vec_ok(h, hs, w, K, esz);
  return esz == 2 ? gate_t<bf16_t>(h, hs, w, bias, N, K, rows, cap, vec, out, st) : gate_t<float>(h, hs, w, bias, N, K, rows, cap, vec, out, st);
}

int lk_router_choice(const void* h, long hs, const void* w, int E, int K, long rows, int top, int groups, int keep, float scale, int score,
                     const float* corr, int gscore, int* experts, float* weights, int esz, hipStream_t st) {
  if (rows <= 0) return 0;
  if (E < 1 || E > kMaxExperts || K < 1 || groups < 1 || groups > 64 || E % groups || keep < 1 || keep > groups || top < 1 || top > kMaxTop ||
      top > (E / groups) * keep || score < 0 || score > 1 || gscore < 0 || gscore > 1)
    return -1;
  const int vec = vec_ok(h, hs, w, K, esz);
  return esz == 2 ? router_t<bf16_t>(h, hs, w, E, K, rows, top, groups, keep, scale, score, corr, gscore, vec, experts, weights, st)
                  : router_t<float>(h, hs, w, E, K, rows, top, groups, keep, scale, score, corr, gscore, vec, experts, weights, st);
}
