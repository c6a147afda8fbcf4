// Linear attention with a fixed decay per head on the matrix cores (bf16 inputs, v_mfma_f32_16x16x32_bf16):
//   S_t = dec S_(t-1) + k_t v_t^T,   o_t = S_t^T q_t        (S [D][V] per sequence and head, fp32)
// in blocks of 64 tokens.  With S the state in front of a block and i, j token numbers inside it,
//   o_i = dec^(i+1) S^T q_i + sum_(j <= i) dec^(i-j) (q_i . k_j) v_j,
//   S  <- dec^n S + sum_j dec^(n-1-j) k_j v_j^T             (n tokens in the block).
// Rows of x (bf16, stride xs): q [H][D] | k [H][D] | v [H][V]; with SILU each through z sigmoid(z), rounded to bf16.
// q, k and v are exact operands then; the decayed scores, the decayed values and the state enter a product as a sum
// of two bf16 numbers (hi + lo: 16 bits and more), and every sum is fp32.
//
// A workgroup of NW waves owns 16 NW value columns of one (item, head); wave w holds the state of its 16 columns in
// accumulators, tile dt: rows d = 16 dt + 4 hq + i, column r (lane = 16 hq + r).  As the second operand of S^T q the
// contraction index may be ordered freely as long as both operands agree, so a chunk of 32 rows is taken in the order
// the accumulators hold it -- slots (hq, 0..3) = rows 4 hq.., slots (hq, 4..7) = rows 16 + 4 hq.. -- and no lane
// exchanges anything.  Scores are formed transposed (keys x queries): a lane then has four neighbouring keys of one
// query, one 8-byte LDS store.  Transposed keys and values (the operands with tokens along the contraction) are
// written 4 x 4 entries at a time; 16-byte granules of a row are permuted by a key of the row (tkey) against bank
// conflicts.  The next block's rows are fetched into registers while the current one is computed.
//
// Segments as in mixer_ops.hip.  MODE 0: an item is a segment, from the slot's state (or zero) to the slot's state.
// MODE 1: an item is a range of a segment ([n][4]: segment, first row, rows, -) from a zero state, its end state goes
// to cs [items][H][D][V];  decay_carry_kernel turns cs into every range's START state and advances the slot;
// MODE 2: the range from its start state, writing o [T][H V] (fp32).
#include "common.h"

namespace k8s {

constexpr int kLaTok = 64;             // tokens per block
constexpr int kLaPad = 8;              // row padding (entries) of the token-major tiles

struct LinArgs {
  const uint16_t* x;
  int xs;
  const float* decay;
  float* state;
  const int* seg_row0;
  const int* seg_pos0;
  const int* seg_slot;
  const int* items;
  float* cs;
  float* o;
  int H, V;
};

// dec^n by repeated squaring
__device__ __forceinline__ float ipow(float dec, int n) {
  float r = 1.f, b = dec;
  for (; n > 0; n >>= 1) {
    if (n & 1) r *= b;
    b *= b;
  }
  return r;
}

// two packed bf16 numbers through z sigmoid(z)
template <bool SILU>
__device__ __forceinline__ uint32_t la_act(uint32_t v) {
  if (!SILU) return v;
  const float a = silu_hw(__uint_as_float(v << 16)), b = silu_hw(__uint_as_float(v & 0xffff0000u));
  return (uint32_t)f2bf(a) | ((uint32_t)f2bf(b) << 16);
}

// entry (row, t) of a transposed tile: rows of 64 tokens, 32 dwords apart, with 32 dwords more every 32 rows
__device__ __forceinline__ int tkey(int row) { return ((row >> 2) ^ (((row >> 1) & 1) << 2)) & 7; }
__device__ __forceinline__ int tofs(int row, int t) {
  return row * 64 + (row >> 5) * 64 + ((((t >> 3) ^ tkey(row)) << 3) | (t & 7));
}
constexpr int trow(int rows) { return rows * 64 + (rows / 32) * 64; }

__device__ __forceinline__ bf16x8 lds16(const uint16_t* p) { return *reinterpret_cast<const bf16x8*>(p); }

// a 4-token x 4-column block of rows t .. t + 3 (zeros past n), two packed words per row
struct Blk {
  uint2 r[4];
};
__device__ __forceinline__ void blk_load(Blk& b, const uint16_t* p, size_t xs, int t, int n) {
#pragma unroll
  for (int k = 0; k < 4; ++k) b.r[k] = t + k < n ? *reinterpret_cast<const uint2*>(p + (t + k) * xs) : uint2{0u, 0u};
}
template <bool SILU>
__device__ __forceinline__ void blk_act(Blk& b) {
#pragma unroll
  for (int k = 0; k < 4; ++k) {
    b.r[k].x = la_act<SILU>(b.r[k].x);
    b.r[k].y = la_act<SILU>(b.r[k].y);
  }
}
__device__ __forceinline__ void blk_rows(const Blk& b, uint16_t* s, int ld, int t, int c) {
#pragma unroll
  for (int k = 0; k < 4; ++k) *reinterpret_cast<uint2*>(s + (t + k) * ld + c) = b.r[k];
}
__device__ __forceinline__ void blk_cols(const Blk& b, uint16_t* s, int t, int c) {
  constexpr uint32_t kLo = 0x05040100u, kHi = 0x07060302u;     // low / high halves of (second : first)
#pragma unroll
  for (int k = 0; k < 4; ++k) {
    const uint32_t sel = (k & 1) ? kHi : kLo;
    const uint32_t w0 = k < 2 ? b.r[0].x : b.r[0].y, w1 = k < 2 ? b.r[1].x : b.r[1].y,
                   w2 = k < 2 ? b.r[2].x : b.r[2].y, w3 = k < 2 ? b.r[3].x : b.r[3].y;
    *reinterpret_cast<uint2*>(s + tofs(c + k, t)) =
        uint2{__builtin_amdgcn_perm(w1, w0, sel), __builtin_amdgcn_perm(w3, w2, sel)};
  }
}

// hi + lo bf16 parts of eight floats
__device__ __forceinline__ void split8(const float (&v)[8], bf16x8& hi, bf16x8& lo) {
#pragma unroll
  for (int j = 0; j < 8; ++j) {
    hi[j] = (__bf16)v[j];
    lo[j] = (__bf16)(v[j] - (float)hi[j]);
  }
}

template <int D, int NW>
constexpr int la_lds_bytes(bool outputs) {
  constexpr int ld = D + kLaPad, k_or_p = kLaTok * ld > 2 * kLaTok * (kLaTok + kLaPad) ? kLaTok * ld
                                                                                         : 2 * kLaTok * (kLaTok + kLaPad);
  return 2 * (trow(D) + trow(16 * NW) + (outputs ? kLaTok * ld + k_or_p : 0));
}

template <int D, int NW, int MODE, bool SILU>
__global__ void __launch_bounds__(64 * NW, 2) decay_attn_mfma_kernel(LinArgs a) {
  constexpr int NT = 64 * NW, VB = 16 * NW, ND = D / 16, NC = D / 32, LD = D + kLaPad, LP = kLaTok + kLaPad;
  constexpr int KB = (16 * (D / 4) + NT - 1) / NT, VBK = (16 * (VB / 4) + NT - 1) / NT;   // blocks per thread
  extern __shared__ __attribute__((aligned(16))) unsigned char lds_raw[];
  __shared__ float pw[kLaTok + 1];
  uint16_t* sKt = reinterpret_cast<uint16_t*>(lds_raw);     // [D][64] transposed
  uint16_t* sVt = sKt + trow(D);                            // [VB][64] transposed
  uint16_t* sQ = sVt + trow(VB);                            // [64][LD]
  uint16_t* sK = sQ + kLaTok * LD;                          // [64][LD]; later the scores, hi and lo [64][LP]
  uint16_t* sPh = sK;
  uint16_t* sPl = sK + kLaTok * LP;
  const int it = blockIdx.x, hh = blockIdx.y, v0 = blockIdx.z * VB, tid = threadIdx.x;
  const int lane = tid & 63, r = lane & 15, hq = lane >> 4;
  const int wv = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int H = a.H, V = a.V;
  int r0, r1;
  bool fresh;
  float* st;
  if (MODE == 0) {
    r0 = a.seg_row0[it];
    r1 = a.seg_row0[it + 1];
    fresh = a.seg_pos0[it] == 0;
    st = a.state + ((size_t)a.seg_slot[it] * H + hh) * D * V;
  } else {
    r0 = a.items[it * 4 + 1];
    r1 = r0 + a.items[it * 4 + 2];
    fresh = MODE == 1;
    st = a.cs + ((size_t)it * H + hh) * D * V;
  }
  const int vcol = v0 + 16 * wv + r;                        // this lane's value column
  const bool vok = v0 + 16 * wv < V;                        // (V % 16 == 0: the whole wave)
  if (tid <= kLaTok) pw[tid] = ipow(a.decay[hh], tid);
  f32x4 S[ND];
#pragma unroll
  for (int dt = 0; dt < ND; ++dt)
#pragma unroll
    for (int i = 0; i < 4; ++i) S[dt][i] = (!fresh && vok) ? st[(size_t)(16 * dt + 4 * hq + i) * V + vcol] : 0.f;
  Blk bq[MODE != 1 ? KB : 1], bk[KB], bv[VBK];
  const int qo = hh * D, ko = (H + hh) * D, vo = 2 * H * D + hh * V + v0;
  auto fetch = [&](int t0) {
    const uint16_t* xp = a.x + (size_t)t0 * a.xs;
    const int n = r1 - t0;
#pragma unroll
    for (int b = 0; b < KB; ++b) {
      const int e = tid + b * NT, t = e / (D / 4) * 4, c = e % (D / 4) * 4;
      if ((16 * (D / 4)) % NT == 0 || t < kLaTok) {
        if (MODE != 1) blk_load(bq[b], xp + qo + c, a.xs, t, n);
        blk_load(bk[b], xp + ko + c, a.xs, t, n);
      }
    }
#pragma unroll
    for (int b = 0; b < VBK; ++b) {
      const int e = tid + b * NT, t = e / (VB / 4) * 4, c = e % (VB / 4) * 4;
      blk_load(bv[b], xp + vo + c, a.xs, t, v0 + c < V ? n : 0);
    }
  };
  fetch(r0);
  for (int t0 = r0; t0 < r1; t0 += kLaTok) {
    const int nb = min(kLaTok, r1 - t0);
    __syncthreads();                                        // the previous block's tiles are read no more
#pragma unroll
    for (int b = 0; b < KB; ++b) {
      const int e = tid + b * NT, t = e / (D / 4) * 4, c = e % (D / 4) * 4;
      if ((16 * (D / 4)) % NT == 0 || t < kLaTok) {
        blk_act<SILU>(bk[b]);
        blk_cols(bk[b], sKt, t, c);
        if (MODE != 1) {
          blk_act<SILU>(bq[b]);
          blk_rows(bk[b], sK, LD, t, c);
          blk_rows(bq[b], sQ, LD, t, c);
        }
      }
    }
#pragma unroll
    for (int b = 0; b < VBK; ++b) {
      const int e = tid + b * NT, t = e / (VB / 4) * 4, c = e % (VB / 4) * 4;
      blk_act<SILU>(bv[b]);
      blk_cols(bv[b], sVt, t, c);
    }
    __syncthreads();
    if (t0 + kLaTok < r1) fetch(t0 + kLaTok);
    f32x4 O[4];
    if (MODE != 1) {
      // scores of the query tile tt against its key tiles (st <= tt), shared out over the waves
      constexpr int SS = NW / 4, NS = 4 / SS;               // key tiles per wave: every SS-th
      const int tt = wv & 3, s0 = wv >> 2;
      f32x4 P[NS];
#pragma unroll
      for (int k = 0; k < NS; ++k) {
        P[k] = f32x4{0.f, 0.f, 0.f, 0.f};
        const int ks = s0 + k * SS;
        if (ks <= tt) {
#pragma unroll
          for (int c = 0; c < NC; ++c)
            P[k] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(lds16(sK + (16 * ks + r) * LD + 32 * c + 8 * hq),
                                                           lds16(sQ + (16 * tt + r) * LD + 32 * c + 8 * hq), P[k], 0, 0, 0);
        }
      }
      // what the state in front of the block gives
#pragma unroll
      for (int t = 0; t < 4; ++t) O[t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int c = 0; c < NC; ++c) {
        float sv[8];
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          sv[i] = S[2 * c][i];
          sv[4 + i] = S[2 * c + 1][i];
        }
        bf16x8 sh, sl;
        split8(sv, sh, sl);
#pragma unroll
        for (int t = 0; t < 4; ++t) {
          const uint16_t* qp = sQ + (16 * t + r) * LD + 32 * c + 4 * hq;
          const bf16x4 q0 = *reinterpret_cast<const bf16x4*>(qp), q1 = *reinterpret_cast<const bf16x4*>(qp + 16);
          const bf16x8 qf = __builtin_shufflevector(q0, q1, 0, 1, 2, 3, 4, 5, 6, 7);
          O[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qf, sh, O[t], 0, 0, 0);
          O[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(qf, sl, O[t], 0, 0, 0);
        }
      }
#pragma unroll
      for (int t = 0; t < 4; ++t)
#pragma unroll
        for (int i = 0; i < 4; ++i) O[t][i] *= pw[16 * t + 4 * hq + i + 1];
      __syncthreads();                                      // every wave is done with sK
#pragma unroll
      for (int k = 0; k < NS; ++k) {
        const int ks = s0 + k * SS;
        if (ks <= (tt | 1)) {                               // a pair of key tiles is read as one chunk: zeros past tt
          u16x4 hi, lo;
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            const int d = 16 * (tt - ks) + r - 4 * hq - i;  // query - key
            const float p = d >= 0 ? P[k][i] * pw[d] : 0.f;
            hi[i] = f2bf(p);
            lo[i] = f2bf(p - bf2f(hi[i]));
          }
          *reinterpret_cast<u16x4*>(sPh + (16 * tt + r) * LP + 16 * ks + 4 * hq) = hi;
          *reinterpret_cast<u16x4*>(sPl + (16 * tt + r) * LP + 16 * ks + 4 * hq) = lo;
        }
      }
      __syncthreads();
    }
    const float dn = pw[nb];
#pragma unroll
    for (int dt = 0; dt < ND; ++dt)
#pragma unroll
      for (int i = 0; i < 4; ++i) S[dt][i] *= dn;
#pragma unroll
    for (int kc = 0; kc < 2; ++kc) {
      const bf16x8 vf = lds16(sVt + tofs(16 * wv + r, 32 * kc + 8 * hq));
      if (MODE != 1) {
#pragma unroll
        for (int t = 2 * kc; t < 4; ++t) {                  // query tiles that see this pair of key tiles
          const int po = (16 * t + r) * LP + 32 * kc + 8 * hq;
          O[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(lds16(sPh + po), vf, O[t], 0, 0, 0);
          O[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(lds16(sPl + po), vf, O[t], 0, 0, 0);
        }
      }
      float vs[8];
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const int e = nb - 1 - (32 * kc + 8 * hq + j);      // (values past the block are zero)
        vs[j] = (float)vf[j] * pw[e > 0 ? e : 0];
      }
      bf16x8 vh, vl;
      split8(vs, vh, vl);
#pragma unroll
      for (int dt = 0; dt < ND; ++dt) {
        const bf16x8 kf = lds16(sKt + tofs(16 * dt + r, 32 * kc + 8 * hq));
        S[dt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, vh, S[dt], 0, 0, 0);
        S[dt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, vl, S[dt], 0, 0, 0);
      }
    }
    if (MODE != 1 && vok) {
#pragma unroll
      for (int t = 0; t < 4; ++t)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int tk = 16 * t + 4 * hq + i;
          if (tk < nb) a.o[(size_t)(t0 + tk) * H * V + (size_t)hh * V + vcol] = O[t][i];
        }
    }
  }
  if (MODE != 2 && vok) {
#pragma unroll
    for (int dt = 0; dt < ND; ++dt)
#pragma unroll
      for (int i = 0; i < 4; ++i) st[(size_t)(16 * dt + 4 * hq + i) * V + vcol] = S[dt][i];
  }
}

// Between the two passes, one thread per state entry of a (segment, head): walk the segment's ranges, replace every
// range's end-from-zero state by its START state, leave the final state in the slot.
__global__ void __launch_bounds__(256) decay_carry_kernel(const float* __restrict__ decay, float* __restrict__ state,
                                                          const int* __restrict__ seg_pos0,
                                                          const int* __restrict__ seg_slot,
                                                          const int* __restrict__ seg_item0,
                                                          const int* __restrict__ items, float* __restrict__ cs, int H,
                                                          int DV) {
  const int sg = blockIdx.x, hh = blockIdx.y, e = blockIdx.z * 256 + threadIdx.x;
  if (e >= DV) return;
  float* st = state + ((size_t)seg_slot[sg] * H + hh) * DV + e;
  float S = seg_pos0[sg] == 0 ? 0.f : *st;
  const float dec = decay[hh];
  for (int k = seg_item0[sg]; k < seg_item0[sg + 1]; ++k) {
    float* ck = cs + ((size_t)k * H + hh) * DV + e;
    const float loc = *ck;
    *ck = S;
    S = fmaf(ipow(dec, items[k * 4 + 2]), S, loc);
  }
  *st = S;
}

template <int D, int NW, int MODE, bool SILU>
static int launch_la(const LinArgs& a, int items, hipStream_t s) {
  constexpr int lds = la_lds_bytes<D, NW>(MODE != 1);
  auto k = decay_attn_mfma_kernel<D, NW, MODE, SILU>;
  if (lds > 48 * 1024 && hipFuncSetAttribute((const void*)k, hipFuncAttributeMaxDynamicSharedMemorySize, lds))
    return (int)hipGetLastError();
  hipLaunchKernelGGL(k, dim3(items, a.H, (a.V + 16 * NW - 1) / (16 * NW)), dim3(64 * NW), lds, s, a);
  return (int)hipGetLastError();
}

template <int D, int NW, bool SILU>
static int launch_la_all(const LinArgs& a, int n_seg, int n_items, const int* seg_item0, hipStream_t s) {
  if (n_items <= 0) return launch_la<D, NW, 0, SILU>(a, n_seg, s);
  int rc = launch_la<D, NW, 1, SILU>(a, n_items, s);
  if (rc) return rc;
  hipLaunchKernelGGL(decay_carry_kernel, dim3(n_seg, a.H, (D * a.V + 255) / 256), dim3(256), 0, s, a.decay, a.state,
                     a.seg_pos0, a.seg_slot, seg_item0, a.items, a.cs, a.H, D * a.V);
  rc = (int)hipGetLastError();
  return rc ? rc : launch_la<D, NW, 2, SILU>(a, n_items, s);
}

template <int D, bool SILU>
static int launch_la_v(const LinArgs& a, int n_seg, int n_items, const int* seg_item0, hipStream_t s) {
  return a.V > 64 ? launch_la_all<D, 8, SILU>(a, n_seg, n_items, seg_item0, s)
                  : launch_la_all<D, 4, SILU>(a, n_seg, n_items, seg_item0, s);
}

}  // namespace k8s

using namespace k8s;

// 1 when the matrix-core kernel takes these sizes (bf16 rows, 8-byte aligned)
K8S_API int k8s_decay_attn_mfma_ok(int D, int V) {
  return (D == 32 || D == 64 || D == 96 || D == 128) && V >= 16 && V % 16 == 0;
}

K8S_API int k8s_decay_attn_mfma(const void* x, int xs, int silu, const float* decay, float* state, const int* seg_row0,
                                const int* seg_pos0, const int* seg_slot, float* o, int n_seg, int H, int D, int V,
                                hipStream_t s, const int* items, int n_items, const int* seg_item0, float* cs) {
  if (n_seg <= 0) return 0;
  if (!k8s_decay_attn_mfma_ok(D, V) || H < 1 || xs % 4 || ((uintptr_t)x & 7) || xs < H * (2 * D + V) ||
      (n_items > 0 && (!items || !seg_item0 || !cs)))
    return (int)hipErrorInvalidValue;
  LinArgs a;
  a.x = (const uint16_t*)x;
  a.xs = xs;
  a.decay = decay;
  a.state = state;
  a.seg_row0 = seg_row0;
  a.seg_pos0 = seg_pos0;
  a.seg_slot = seg_slot;
  a.items = items;
  a.cs = cs;
  a.o = o;
  a.H = H;
  a.V = V;
#define K8S_LA(DD)                                                                    \
  return silu ? launch_la_v<DD, true>(a, n_seg, n_items, seg_item0, s)                \
              : launch_la_v<DD, false>(a, n_seg, n_items, seg_item0, s)
  switch (D) {
    case 32: K8S_LA(32);
    case 64: K8S_LA(64);
    case 96: K8S_LA(96);
    default: K8S_LA(128);
  }
#undef K8S_LA
}
