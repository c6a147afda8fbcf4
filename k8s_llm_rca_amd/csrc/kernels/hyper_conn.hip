// Hyper-connections: S copies ("streams") of the fp32 residual around every sublayer.
//
// The streams lie [T][S][W].  A sublayer reads  u = sum_s in[s] x_s, RMS-normed; its output y goes back as
//   x_r <- sum_s mix[s][r] x_s + out[r] y        (all r at once from the old streams; mix is [from][to]).
// The write-back of one sublayer and the read of the next are ONE pass: every stream is read and written once,
// and the next sublayer's normed input leaves the same pass as activations (TA: bf16 as uint16_t, or float).
// The output of a mixture of experts is joined on the way in: y = sum_k w[t][k] yp[inv[t K + k]], the rows of
// the experts' outputs in expert order, so the joined fp32 row is never written.
// S = 1 with in = mix = 1 is the plain pre-norm residual.
// A step may also add the embedding output once more on the way (x_r += escale * embed[eid[t]] for every stream):
// stacks of layers that run several times in a row read it again in front of every further pass.
//
// One workgroup per row; a thread owns VEC neighbouring columns of all streams, so the S x S mix is in
// registers; the row of u stays in LDS between the sum of squares and the output.
#include "common.h"

namespace k8s {

template <int VEC, typename T>
__device__ __forceinline__ void ldv(const T* p, size_t i, float (&v)[VEC]);
template <>
__device__ __forceinline__ void ldv<1, float>(const float* p, size_t i, float (&v)[1]) { v[0] = p[i]; }
template <>
__device__ __forceinline__ void ldv<1, uint16_t>(const uint16_t* p, size_t i, float (&v)[1]) { v[0] = bf2f(p[i]); }
template <>
__device__ __forceinline__ void ldv<4, float>(const float* p, size_t i, float (&v)[4]) {
  const f32x4 a = *reinterpret_cast<const f32x4*>(p + i);
#pragma unroll
  for (int k = 0; k < 4; ++k) v[k] = a[k];
}
template <>
__device__ __forceinline__ void ldv<4, uint16_t>(const uint16_t* p, size_t i, float (&v)[4]) {
  const u16x4 a = *reinterpret_cast<const u16x4*>(p + i);
#pragma unroll
  for (int k = 0; k < 4; ++k) v[k] = bf2f(a[k]);
}
template <int VEC, typename T>
__device__ __forceinline__ void stv(T* p, size_t i, const float (&v)[VEC]);
template <>
__device__ __forceinline__ void stv<1, float>(float* p, size_t i, const float (&v)[1]) { p[i] = v[0]; }
template <>
__device__ __forceinline__ void stv<1, uint16_t>(uint16_t* p, size_t i, const float (&v)[1]) { p[i] = f2bf(v[0]); }
template <>
__device__ __forceinline__ void stv<4, float>(float* p, size_t i, const float (&v)[4]) {
  *reinterpret_cast<f32x4*>(p + i) = f32x4{v[0], v[1], v[2], v[3]};
}
template <>
__device__ __forceinline__ void stv<4, uint16_t>(uint16_t* p, size_t i, const float (&v)[4]) {
  *reinterpret_cast<u16x4*>(p + i) = u16x4{f2bf(v[0]), f2bf(v[1]), f2bf(v[2]), f2bf(v[3])};
}

// the row of u (LDS) -> u / sqrt(mean(u^2) + eps) * w as activations; ss: this thread's share of sum(u^2)
template <int VEC, typename TA>
__device__ __forceinline__ void norm_row(const float* u, float ss, float* red, const float* __restrict__ w, float eps,
                                         TA* __restrict__ h, size_t o, int W) {
  const float r = 1.f / sqrtf(block_sum(ss, red) / (float)W + eps);
  for (int c = threadIdx.x * VEC; c < W; c += blockDim.x * VEC) {    // the columns this thread wrote itself
    float wv[VEC], v[VEC];
    ldv<VEC>(w, c, wv);
#pragma unroll
    for (int k = 0; k < VEC; ++k) v[k] = u[c + k] * r * wv[k];
    stv<VEC>(h, o + c, v);
  }
}

constexpr int kMaxStreams = 16;   // the form for any count: one column per thread, the streams in a local array

// S streams at compile time (S > 0) or S_ <= kMaxStreams of them (S == 0).
// y: fp32 rows [T][W], or (inv given) rows of yp in expert order weighted by ew [T][K].
// out / mix: this sublayer's; in / nw: the next one's (h null: nothing reads the streams next).
// eid (optional) [T]: token ids whose rows of emb, times es, are added to every stream.
template <int S, int VEC, typename TY, typename TA>
__global__ void __launch_bounds__(1024) hyper_step_kernel(float* __restrict__ x, const TY* __restrict__ y,
                                                         const int* __restrict__ inv, const float* __restrict__ ew,
                                                         int K, const float* __restrict__ out,
                                                         const float* __restrict__ mix, const float* __restrict__ in,
                                                         const float* __restrict__ nw, float eps, TA* __restrict__ h,
                                                         int W, int S_, const int* __restrict__ eid,
                                                         const TA* __restrict__ emb, float es) {
  extern __shared__ float u[];
  __shared__ float red[16];
  constexpr int SM = S > 0 ? S : kMaxStreams;
  const int n = S > 0 ? S : S_;
  const size_t t = blockIdx.x, o = t * W;
  float* xr = x + o * n;
  const size_t e0 = eid ? (size_t)eid[t] * W : 0;
  float ss = 0.f;
  for (int c = threadIdx.x * VEC; c < W; c += blockDim.x * VEC) {
    float xv[SM][VEC], yv[VEC];
#pragma unroll
    for (int s = 0; s < SM; ++s)
      if (s < n) ldv<VEC>(xr, (size_t)s * W + c, xv[s]);
    if (inv) {
#pragma unroll
      for (int k = 0; k < VEC; ++k) yv[k] = 0.f;
      for (int j = 0; j < K; ++j) {
        float ev[VEC];
        const float wj = ew[t * K + j];
        ldv<VEC>(y, (size_t)inv[t * K + j] * W + c, ev);
#pragma unroll
        for (int k = 0; k < VEC; ++k) yv[k] = fmaf(wj, ev[k], yv[k]);
      }
    } else {
      ldv<VEC>(y, o + c, yv);
    }
    float uv[VEC], av[VEC];
#pragma unroll
    for (int k = 0; k < VEC; ++k) uv[k] = av[k] = 0.f;
    if (eid) ldv<VEC>(emb, e0 + c, av);
#pragma unroll
    for (int r = 0; r < SM; ++r)
      if (r < n) {
        float nv[VEC];
        const float orr = out[r];
#pragma unroll
        for (int k = 0; k < VEC; ++k) nv[k] = orr * yv[k];
#pragma unroll
        for (int s = 0; s < SM; ++s)
          if (s < n) {
            const float m = mix[s * n + r];
#pragma unroll
            for (int k = 0; k < VEC; ++k) nv[k] = fmaf(m, xv[s][k], nv[k]);
          }
        if (eid) {
#pragma unroll
          for (int k = 0; k < VEC; ++k) nv[k] = fmaf(es, av[k], nv[k]);
        }
        stv<VEC>(xr, (size_t)r * W + c, nv);
        if (h) {
          const float ir = in[r];
#pragma unroll
          for (int k = 0; k < VEC; ++k) uv[k] = fmaf(ir, nv[k], uv[k]);
        }
      }
    if (h) {
#pragma unroll
      for (int k = 0; k < VEC; ++k) {
        u[c + k] = uv[k];
        ss = fmaf(uv[k], uv[k], ss);
      }
    }
  }
  if (h) norm_row<VEC>(u, ss, red, nw, eps, h, o, W);
}

// x_s = embed[id] * scale for every stream s; h = the first sublayer's normed input.
template <int VEC, typename TE, typename TA>
__global__ void __launch_bounds__(1024) hyper_embed_kernel(const int* __restrict__ ids, const TE* __restrict__ embed,
                                                          float scale, float* __restrict__ x, int S,
                                                          const float* __restrict__ in, const float* __restrict__ nw,
                                                          float eps, TA* __restrict__ h, int W) {
  extern __shared__ float u[];
  __shared__ float red[16];
  const size_t t = blockIdx.x, e0 = (size_t)ids[t] * W;
  float si = 0.f;
  for (int s = 0; s < S; ++s) si += in[s];
  float ss = 0.f;
  for (int c = threadIdx.x * VEC; c < W; c += blockDim.x * VEC) {
    float v[VEC];
    ldv<VEC>(embed, e0 + c, v);
#pragma unroll
    for (int k = 0; k < VEC; ++k) v[k] *= scale;
    for (int s = 0; s < S; ++s) stv<VEC>(x, (t * S + s) * W + c, v);
#pragma unroll
    for (int k = 0; k < VEC; ++k) {
      u[c + k] = si * v[k];
      ss = fmaf(u[c + k], u[c + k], ss);
    }
  }
  norm_row<VEC>(u, ss, red, nw, eps, h, t * W, W);
}

// h = rms(sum_s in[s] x_s) * nw of the given rows (in null: the plain sum).
template <int VEC, typename TA>
__global__ void __launch_bounds__(1024) hyper_read_kernel(const float* __restrict__ x, const int* __restrict__ rows, int S,
                                                         const float* __restrict__ in, const float* __restrict__ nw,
                                                         float eps, TA* __restrict__ h, int W) {
  extern __shared__ float u[];
  __shared__ float red[16];
  const size_t t = rows ? (size_t)rows[blockIdx.x] : blockIdx.x;
  float ss = 0.f;
  for (int c = threadIdx.x * VEC; c < W; c += blockDim.x * VEC) {
    float uv[VEC];
#pragma unroll
    for (int k = 0; k < VEC; ++k) uv[k] = 0.f;
    for (int s = 0; s < S; ++s) {
      float v[VEC];
      const float f = in ? in[s] : 1.f;
      ldv<VEC>(x, (t * S + s) * W + c, v);
#pragma unroll
      for (int k = 0; k < VEC; ++k) uv[k] = fmaf(f, v[k], uv[k]);
    }
#pragma unroll
    for (int k = 0; k < VEC; ++k) {
      u[c + k] = uv[k];
      ss = fmaf(uv[k], uv[k], ss);
    }
  }
  norm_row<VEC>(u, ss, red, nw, eps, h, (size_t)blockIdx.x * W, W);
}

// threads per row: few rows (decoding) leave most of the chip idle, so a row gets a thread per VEC columns
static int hyper_threads(int rows, int W, int vec) {
  const int want = ((W + vec - 1) / vec + 63) / 64 * 64;
  const int most = rows <= 256 ? 1024 : 256;
  return want < 64 ? 64 : (want > most ? most : want);
}
static bool hyper_row_ok(int W) { return W > 0 && (size_t)W * sizeof(float) <= 64 * 1024; }

template <int VEC, typename TY, typename TA>
static void hyper_step_launch(float* x, const void* y, const int* inv, const float* ew, int K, const float* out,
                              const float* mix, const float* in, const float* nw, float eps, void* h, int T, int S,
                              int W, const int* eid, const void* emb, float es, hipStream_t s) {
  const dim3 g(T), b(hyper_threads(T, W, VEC));
#define K8S_HS(SS)                                                                                              \
  hipLaunchKernelGGL((hyper_step_kernel<SS, VEC, TY, TA>), g, b, W * sizeof(float), s, x, (const TY*)y, inv, ew, K, \
                     out, mix, in, nw, eps, (TA*)h, W, S, eid, (const TA*)emb, es)
  switch (S) {
    case 1: K8S_HS(1); break;
    case 2: K8S_HS(2); break;
    case 3: K8S_HS(3); break;
    case 4: K8S_HS(4); break;
    default: K8S_HS(0); break;
  }
#undef K8S_HS
}

}  // namespace k8s

using namespace k8s;

// ydt / hdt / edt: 0 bf16, 1 fp32.  inv null: y is fp32 [T][W].  emb has the type of h.
K8S_API int k8s_hyper_step(float* x, const void* y, int ydt, const int* inv, const float* ew, int K, const float* out,
                           const float* mix, const float* in, const float* nw, float eps, void* h, int hdt, int T, int S,
                           int W, hipStream_t s, const int* eid, const void* emb, float es) {
  if (T <= 0) return 0;
  if (!hyper_row_ok(W) || S < 1 || S > kMaxStreams || !y || !out || !mix || (h && (!in || !nw)) ||
      (inv && (!ew || K < 1)) || (!inv && ydt != 1) || (eid && !emb))
    return (int)hipErrorInvalidValue;
#define K8S_HY(VEC)                                                                                               \
  if (ydt == 0 && hdt == 0)                                                                                       \
    hyper_step_launch<VEC, uint16_t, uint16_t>(x, y, inv, ew, K, out, mix, in, nw, eps, h, T, S, W, eid, emb, es, s);             \
  else if (ydt == 0)                                                                                              \
    hyper_step_launch<VEC, uint16_t, float>(x, y, inv, ew, K, out, mix, in, nw, eps, h, T, S, W, eid, emb, es, s);                \
  else if (hdt == 0)                                                                                              \
    hyper_step_launch<VEC, float, uint16_t>(x, y, inv, ew, K, out, mix, in, nw, eps, h, T, S, W, eid, emb, es, s);                \
  else                                                                                                            \
    hyper_step_launch<VEC, float, float>(x, y, inv, ew, K, out, mix, in, nw, eps, h, T, S, W, eid, emb, es, s)
  if (W % 4 == 0 && S <= 4) {
    K8S_HY(4);
  } else {
    K8S_HY(1);
  }
#undef K8S_HY
  return (int)hipGetLastError();
}

K8S_API int k8s_hyper_embed(const int* ids, const void* embed, int edt, float scale, float* x, int S, const float* in,
                            const float* nw, float eps, void* h, int hdt, int T, int W, hipStream_t s) {
  if (T <= 0) return 0;
  if (!hyper_row_ok(W) || S < 1 || !in || !nw || !h) return (int)hipErrorInvalidValue;
#define K8S_HE(VEC, TE, TA)                                                                                       \
  hipLaunchKernelGGL((hyper_embed_kernel<VEC, TE, TA>), dim3(T), dim3(hyper_threads(T, W, VEC)), W * sizeof(float), \
                     s, ids, (const TE*)embed, scale, x, S, in, nw, eps, (TA*)h, W)
#define K8S_HEV(TE, TA)        \
  if (W % 4 == 0) {            \
    K8S_HE(4, TE, TA);         \
  } else {                     \
    K8S_HE(1, TE, TA);         \
  }
  if (edt == 0 && hdt == 0) {
    K8S_HEV(uint16_t, uint16_t)
  } else if (edt == 0) {
    K8S_HEV(uint16_t, float)
  } else if (hdt == 0) {
    K8S_HEV(float, uint16_t)
  } else {
    K8S_HEV(float, float)
  }
#undef K8S_HEV
#undef K8S_HE
  return (int)hipGetLastError();
}

K8S_API int k8s_hyper_read(const float* x, const int* rows, int R, int S, const float* in, const float* nw, float eps,
                           void* h, int hdt, int W, hipStream_t s) {
  if (R <= 0) return 0;
  if (!hyper_row_ok(W) || S < 1 || !nw || !h) return (int)hipErrorInvalidValue;
#define K8S_HR(VEC, TA)                                                                                          \
  hipLaunchKernelGGL((hyper_read_kernel<VEC, TA>), dim3(R), dim3(hyper_threads(R, W, VEC)), W * sizeof(float), s, x, \
                     rows, S, in, nw, eps, (TA*)h, W)
  if (W % 4 == 0 && hdt == 0) {
    K8S_HR(4, uint16_t);
  } else if (W % 4 == 0) {
    K8S_HR(4, float);
  } else if (hdt == 0) {
    K8S_HR(1, uint16_t);
  } else {
    K8S_HR(1, float);
  }
#undef K8S_HR
  return (int)hipGetLastError();
}
