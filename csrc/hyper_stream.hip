// A residual stream kept as S mixed copies X_s (f32), one sublayer boundary per pass over a token's copies:
//
//   r   = a + b + sum_k yw[t, k] y[t top + k]              the sublayer's result (dense rows, weighted expert rows)
//   X_t <- sum_s mix[s, t] X_s + wout[t] r                 all t at once from the old copies
//   u   = sum_s win[s] X_s                                 the next sublayer's combination (win null: the sum)
//   out = (u - mean) / sqrt(mean((u - mean)^2) + eps) * w * oscale
//
// The copies may all be equal still (one [T, W] tensor read with stream stride 0); the first update then writes them out.
// Beside it: the square of relu in place.  bf16 or f32 activations; everything between the loads and the stores is f32.
#include "common.h"
#include "kernels.h"

namespace {

template <typename T>
LK_DEVICE float ldv(const T* p);
template <>
LK_DEVICE float ldv<bf16_t>(const bf16_t* p) { return bf2f(*p); }
template <>
LK_DEVICE float ldv<float>(const float* p) { return *p; }
template <typename T>
LK_DEVICE void stv(T* p, float v);
template <>
LK_DEVICE void stv<bf16_t>(bf16_t* p, float v) { *p = f2bf(v); }
template <>
LK_DEVICE void stv<float>(float* p, float v) { *p = v; }

template <typename T, int V>
LK_DEVICE void ldn(const T* p, float (&f)[V]) {
  if constexpr (V == 4 && sizeof(T) == 4) {
    const floatx4 t = *reinterpret_cast<const floatx4*>(p);
#pragma unroll
    for (int e = 0; e < 4; ++e) f[e] = t[e];
  } else if constexpr (V == 4) {
    const short4_t t = *reinterpret_cast<const short4_t*>(p);
#pragma unroll
    for (int e = 0; e < 4; ++e) f[e] = bf2f((bf16_t)t[e]);
  } else {
    f[0] = ldv<T>(p);
  }
}

template <typename T, int V>
LK_DEVICE void stn(T* p, const float (&f)[V]) {
  if constexpr (V == 4 && sizeof(T) == 4) {
    *reinterpret_cast<floatx4*>(p) = floatx4{f[0], f[1], f[2], f[3]};
  } else if constexpr (V == 4) {
    *reinterpret_cast<short4_t*>(p) = short4_t{(short)f2bf(f[0]), (short)f2bf(f[1]), (short)f2bf(f[2]), (short)f2bf(f[3])};
  } else {
    stv<T>(p, f[0]);
  }
}

struct HyperParams {
  const float* xin;   // row t, copy s: xin + t * xrow + s * xstr
  long xrow, xstr;
  float* xout;        // [T, S, W]; null: no update
  const void* a;
  long as;
  const void* b;
  long bs;
  const void* y;
  long ys;
  const float* yw;
  int top;
  const float* mix;   // [S, S], from x to
  const float* wout;  // [S]
  const float* win;   // [S] or null
  const float* w;     // [W] or null: no normed copy
  float eps, oscale;
  const long* idx;    // rows to norm (no update); null: every row
  void* out;
  long os;
  int S, W;
};

// One workgroup per token; thread i owns the column groups i, i + 256, ... of V adjacent columns: per group the SM copies are in
// registers from the load to the store, and the combination u stays there (MAXI groups) for the two reductions of the norm.
template <typename T, int SM, int MAXI, int V>
__global__ __launch_bounds__(256) void stream_hyper_norm_kernel(HyperParams p) {
  __shared__ float red[4];
  const long row = blockIdx.x, src = p.idx ? p.idx[row] : row;
  const int ng = p.W / V;
  const T* a = reinterpret_cast<const T*>(p.a);
  const T* b = reinterpret_cast<const T*>(p.b);
  const T* y = reinterpret_cast<const T*>(p.y);
  const bool upd = p.xout != nullptr;
  float mix[SM][SM], wo[SM], wi[SM];
#pragma unroll
  for (int s = 0; s < SM; ++s) {
    const bool in = s < p.S;
    wi[s] = in ? (p.win ? p.win[s] : 1.f) : 0.f;
    wo[s] = upd && in ? p.wout[s] : 0.f;
#pragma unroll
    for (int t = 0; t < SM; ++t) mix[s][t] = upd && in && t < p.S ? p.mix[s * p.S + t] : 0.f;
  }
  float u[MAXI][V];
  float sum = 0.f;
#pragma unroll
  for (int i = 0; i < MAXI; ++i) {
    const int c = (threadIdx.x + 256 * i) * V;
#pragma unroll
    for (int e = 0; e < V; ++e) u[i][e] = 0.f;
    if (threadIdx.x + 256 * i < ng) {
      float x[SM][V];
#pragma unroll
      for (int s = 0; s < SM; ++s) {
        if (s < p.S) {
          ldn<float, V>(p.xin + src * p.xrow + s * p.xstr + c, x[s]);
        } else {
#pragma unroll
          for (int e = 0; e < V; ++e) x[s][e] = 0.f;
        }
      }
      if (upd) {
        float r[V], t[V];
#pragma unroll
        for (int e = 0; e < V; ++e) r[e] = 0.f;
        if (a) {
          ldn<T, V>(a + row * p.as + c, t);
#pragma unroll
          for (int e = 0; e < V; ++e) r[e] += t[e];
        }
        if (b) {
          ldn<T, V>(b + row * p.bs + c, t);
#pragma unroll
          for (int e = 0; e < V; ++e) r[e] += t[e];
        }
        if (y) {
          for (int k = 0; k < p.top; ++k) {
            const float wk = p.yw[row * p.top + k];
            ldn<T, V>(y + (row * p.top + k) * p.ys + c, t);
#pragma unroll
            for (int e = 0; e < V; ++e) r[e] += wk * t[e];
          }
        }
        float n[SM][V];
#pragma unroll
        for (int d = 0; d < SM; ++d)
#pragma unroll
          for (int e = 0; e < V; ++e) {
            float v = wo[d] * r[e];
#pragma unroll
            for (int s = 0; s < SM; ++s) v += mix[s][d] * x[s][e];
            n[d][e] = v;
          }
#pragma unroll
        for (int d = 0; d < SM; ++d) {
          if (d < p.S) stn<float, V>(p.xout + (row * p.S + d) * p.W + c, n[d]);
#pragma unroll
          for (int e = 0; e < V; ++e) x[d][e] = n[d][e];
        }
      }
#pragma unroll
      for (int e = 0; e < V; ++e) {
#pragma unroll
        for (int s = 0; s < SM; ++s) u[i][e] += wi[s] * x[s][e];
        sum += u[i][e];
      }
    }
  }
  if (!p.out) return;
  const float mean = block_sum<4>(sum, red) / (float)p.W;
  float q = 0.f;
#pragma unroll
  for (int i = 0; i < MAXI; ++i)
    if (threadIdx.x + 256 * i < ng) {
#pragma unroll
      for (int e = 0; e < V; ++e) {
        u[i][e] -= mean;
        q += u[i][e] * u[i][e];
      }
    }
  const float inv = p.oscale / sqrtf(block_sum<4>(q, red) / (float)p.W + p.eps);
#pragma unroll
  for (int i = 0; i < MAXI; ++i) {
    const int c = (threadIdx.x + 256 * i) * V;
    if (threadIdx.x + 256 * i < ng) {
      float wv[V], r[V];
      ldn<float, V>(p.w + c, wv);
#pragma unroll
      for (int e = 0; e < V; ++e) r[e] = u[i][e] * inv * wv[e];
      stn<T, V>(reinterpret_cast<T*>(p.out) + row * p.os + c, r);
    }
  }
}

template <typename T, int SM>
int hyper_s(const HyperParams& p, long rows, bool vec, hipStream_t st) {
#define LK_HYPER(MAXI, V) stream_hyper_norm_kernel<T, SM, MAXI, V><<<(unsigned)rows, 256, 0, st>>>(p)
  if (vec && p.W <= 1024) LK_HYPER(1, 4);
  else if (vec && p.W <= 2048) LK_HYPER(2, 4);
  else if (vec && p.W <= 4096) LK_HYPER(4, 4);
  else if (vec && p.W <= 8192) LK_HYPER(8, 4);
  else if (p.W <= 4096) LK_HYPER(16, 1);
  else return -1;
#undef LK_HYPER
  LK_CHECK_LAUNCH();
  return 0;
}

template <typename T>
int hyper_t(const HyperParams& p, long rows, bool vec, hipStream_t st) {
  if (p.S <= 2) return hyper_s<T, 2>(p, rows, vec, st);
  if (p.S <= 4) return hyper_s<T, 4>(p, rows, vec, st);
  return hyper_s<T, 8>(p, rows, vec, st);
}

template <typename T, int V>
__global__ __launch_bounds__(256) void relu_sq_kernel(T* __restrict__ x, long xs, int n) {
  const long t = blockIdx.x;
  for (int c = (blockIdx.y * 256 + threadIdx.x) * V; c < n; c += 256 * V * gridDim.y) {
    float f[V];
    ldn<T, V>(x + t * xs + c, f);
#pragma unroll
    for (int e = 0; e < V; ++e) {
      const float r = fmaxf(f[e], 0.f);
      f[e] = r * r;
    }
    stn<T, V>(x + t * xs + c, f);
  }
}

}  // namespace

int lk_stream_hyper_norm(const float* xin, long xrow, long xstr, float* xout, int S, const void* a, long as, const void* b, long bs,
                         const void* y, long ys, const float* yw, int top, const float* mix, const float* wout, const float* win,
                         const float* w, float eps, float oscale, const long* idx, void* out, long os, long rows, int W, int esz,
                         hipStream_t st) {
  if (rows <= 0) return 0;
  if (S < 1 || S > 8 || W < 1 || (y && (!yw || top < 1)) || (out && !w) || (xout && (idx || !mix || !wout)) || (!xout && !out)) return -1;
  const auto al = [](const void* p, long stride_bytes, int vec_bytes) {
    return p == nullptr || (reinterpret_cast<uintptr_t>(p) % vec_bytes == 0 && stride_bytes % vec_bytes == 0);
  };
  const int tv = esz == 2 ? 8 : 16;
  const bool vec = W % 4 == 0 && al(xin, xrow * 4, 16) && xstr % 4 == 0 && al(xout, 0, 16) && al(w, 0, 16) && al(a, as * (long)esz, tv) &&
                   al(b, bs * (long)esz, tv) && al(y, ys * (long)esz, tv) && al(out, os * (long)esz, tv);
  HyperParams p;
  p.xin = xin; p.xrow = xrow; p.xstr = xstr; p.xout = xout; p.a = a; p.as = as; p.b = b; p.bs = bs; p.y = y; p.ys = ys; p.yw = yw;
  p.top = top; p.mix = mix; p.wout = wout; p.win = win; p.w = w; p.eps = eps; p.oscale = oscale; p.idx = idx; p.out = out; p.os = os;
  p.S = S; p.W = W;
  return esz == 2 ? hyper_t<bf16_t>(p, rows, vec, st) : hyper_t<float>(p, rows, vec, st);
}

int lk_relu_sq_(void* x, long xs, long rows, int n, int esz, hipStream_t st) {
  if (rows <= 0 || n <= 0) return 0;
  const bool vec = n % 4 == 0 && xs % 4 == 0 && reinterpret_cast<uintptr_t>(x) % (4 * esz) == 0;
  const int per = vec ? 1024 : 256;
  const dim3 grid((unsigned)rows, (unsigned)((n + per - 1) / per < 64 ? (n + per - 1) / per : 64));
  if (esz == 2) {
    if (vec) relu_sq_kernel<bf16_t, 4><<<grid, 256, 0, st>>>((bf16_t*)x, xs, n);
    else relu_sq_kernel<bf16_t, 1><<<grid, 256, 0, st>>>((bf16_t*)x, xs, n);
  } else {
    if (vec) relu_sq_kernel<float, 4><<<grid, 256, 0, st>>>((float*)x, xs, n);
    else relu_sq_kernel<float, 1><<<grid, 256, 0, st>>>((float*)x, xs, n);
  }
  LK_CHECK_LAUNCH();
  return 0;
}
