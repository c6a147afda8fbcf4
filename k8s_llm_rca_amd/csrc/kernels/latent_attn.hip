// Attention over a paged LATENT cache (one vector of R numbers per token, shared
// by every head): the keys' and values' up-projections are moved to the query and
// output side, so a head's query is qa[h] = W_uk[h]^T q[h] (R numbers), its
// score against token j is scale * qa[h] . c_j, and its output in latent space
// is sum_j p_j c_j; the caller applies W_uv[h] afterwards.  All heads of a token
// read the same keys once.  Causal softmax in fp32; the optional per-head output gate
// sigmoid(gate[t][h]) is applied here (it commutes with W_uv).
//
// A cache row may hold RP more numbers behind the latent, a key part shared by all heads (the rotated
// one): a head's query then has RP more entries qr[t][h] and the score is scale * (qa[h] . c_j + qr[h] . k_j);
// the values stay the latents alone.  window > 0: position i sees j with i - j < window.  sink (optional) [H]:
// exp(sink_h) is added to head h's denominator, without a key or a value.
//
// Rows are addressed through the step's segments (seq_ops.hip): row r of segment
// s is the token at position seg_pos0[s] + r - seg_row0[s] and sees keys 0 .. that
// position, read through block table row s ([n_seg][maxb] pages of BS tokens).
#include "common.h"

namespace k8s {

template <typename T>
__device__ __forceinline__ float ldc(const T* p, size_t i);
template <>
__device__ __forceinline__ float ldc<float>(const float* p, size_t i) { return p[i]; }
template <>
__device__ __forceinline__ float ldc<uint16_t>(const uint16_t* p, size_t i) { return bf2f(p[i]); }
template <typename T>
__device__ __forceinline__ void sto(T* p, size_t i, float v);
template <>
__device__ __forceinline__ void sto<float>(float* p, size_t i, float v) { p[i] = v; }
template <>
__device__ __forceinline__ void sto<uint16_t>(uint16_t* p, size_t i, float v) { p[i] = f2bf(v); }

constexpr int kKT = 32;       // keys per tile
constexpr int kMaxAcc = 8;    // outputs per thread and head group

// Any H and R, fp32 arithmetic on the vector pipes: the reference form (fp32
// models, and shapes the MFMA kernels do not take).  One workgroup per row;
// heads in groups of HG with HG * R <= 256 * kMaxAcc.
// LDS: q[HG][W] | ct[kKT][W + 1] | sc[HG][kKT] | m[HG] l[HG] al[HG]   (W = R + RP: a cache row)
// qa is addressed qa[t * qst + h * qsh + c], out likewise with ost / osh; qr is [T][H][RP].
template <typename TC, typename TO>
__global__ void __launch_bounds__(256) latent_attn_rows_kernel(
    const float* __restrict__ qa, const TC* __restrict__ cache, const int* __restrict__ bt, int maxb,
    const int* __restrict__ row_seg, const int* __restrict__ seg_row0, const int* __restrict__ seg_pos0,
    const float* __restrict__ gate, int ldg, TO* __restrict__ out, int row_base, int H, int R, int BS, int HG,
    float scale, long qst, long qsh, const float* __restrict__ qr, int RP, long ost, long osh, int window,
    const float* __restrict__ sink) {
  extern __shared__ float smem[];
  const int W = R + RP;
  float* q = smem;
  float* ct = q + HG * W;
  float* sc = ct + kKT * (W + 1);
  float* m = sc + HG * kKT;
  float* l = m + HG;
  float* al = l + HG;
  const int r = row_base + blockIdx.x, tid = threadIdx.x, lane = tid & 63, wv = tid >> 6;
  const int sg = row_seg[r];
  const int ctx = seg_pos0[sg] + (r - seg_row0[sg]) + 1;
  const int klo = window > 0 ? max(0, ctx - window) : 0;     // the first key this row sees
  const int* pages = bt + (size_t)sg * maxb;
  for (int h0 = 0; h0 < H; h0 += HG) {
    const int hg = min(HG, H - h0), no = hg * R;
    for (int i = tid; i < hg * W; i += 256) {
      const int h = i / W, c = i - h * W;
      q[i] = c < R ? qa[r * qst + (h0 + h) * qsh + c] : qr[((size_t)r * H + h0 + h) * RP + c - R];
    }
    if (tid < hg) {
      m[tid] = sink ? sink[h0 + tid] : -INFINITY;
      l[tid] = sink ? 1.f : 0.f;
    }
    float acc[kMaxAcc];
#pragma unroll
    for (int i = 0; i < kMaxAcc; ++i) acc[i] = 0.f;
    for (int k0 = klo; k0 < ctx; k0 += kKT) {
      const int nk = min(kKT, ctx - k0);
      __syncthreads();
      for (int i = tid; i < kKT * W; i += 256) {
        const int j = i / W, c = i - j * W, kp = k0 + j;
        float v = 0.f;
        if (j < nk) v = ldc(cache, ((size_t)pages[kp / BS] * BS + kp % BS) * W + c);
        ct[j * (W + 1) + c] = v;
      }
      __syncthreads();
      for (int i = tid; i < hg * kKT; i += 256) {
        const int h = i / kKT, j = i - h * kKT;
        float s = -INFINITY;
        if (j < nk) {
          s = 0.f;
          const float* qh = q + h * W;
          const float* cj = ct + j * (W + 1);
          for (int c = 0; c < W; ++c) s = fmaf(qh[c], cj[c], s);
          s *= scale;
        }
        sc[i] = s;
      }
      __syncthreads();
      for (int h = wv; h < hg; h += 4) {      // one wave per head: kKT <= 64 scores
        const float s = lane < kKT ? sc[h * kKT + lane] : -INFINITY;
        const float mo = m[h], mn = fmaxf(mo, wave_max(s));
        const float p = lane < nk ? expf(s - mn) : 0.f;
        const float ps = wave_sum(p);
        if (lane < kKT) sc[h * kKT + lane] = p;
        if (lane == 0) {
          const float a = expf(mo - mn);      // 0 on the first tile (mo = -inf)
          al[h] = a;
          l[h] = l[h] * a + ps;
          m[h] = mn;
        }
      }
      __syncthreads();
#pragma unroll
      for (int i = 0; i < kMaxAcc; ++i) {
        const int o = tid + i * 256;
        if (o < no) {
          const int h = o / R, c = o - h * R;
          float a = acc[i] * al[h];
          const float* ph = sc + h * kKT;
          for (int j = 0; j < nk; ++j) a = fmaf(ph[j], ct[j * (W + 1) + c], a);
          acc[i] = a;
        }
      }
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < kMaxAcc; ++i) {
      const int o = tid + i * 256;
      if (o < no) {
        const int h = o / R, c = o - h * R;
        const float g = gate ? 1.f / (1.f + expf(-gate[(size_t)r * ldg + h0 + h])) : 1.f;
        sto(out, r * ost + (h0 + h) * osh + c, acc[i] / l[h] * g);
      }
    }
    __syncthreads();
  }
}

}  // namespace k8s

using namespace k8s;

// Rows row_base .. row_base + n_rows of the step.  dt: 0 = bf16 cache and output, 1 = fp32.
K8S_API int k8s_latent_attn_rows(const float* qa, const void* cache, const int* bt, int maxb, const int* row_seg,
                                 const int* seg_row0, const int* seg_pos0, const float* gate, int ldg, void* out,
                                 int row_base, int n_rows, int H, int R, int BS, float scale, int dt,
                                 hipStream_t s, long qst, long qsh, const float* qr, int RP, long ost, long osh,
                                 int window, const float* sink) {
  if (n_rows <= 0) return 0;
  if (H <= 0 || R <= 0 || R > 256 * kMaxAcc || RP < 0 || (RP && !qr) || window < 0) return (int)hipErrorInvalidValue;
  int HG = (256 * kMaxAcc) / R;
  if (HG > 64) HG = 64;
  if (HG > H) HG = H;
  const size_t lds = sizeof(float) * ((size_t)HG * (R + RP) + (size_t)kKT * (R + RP + 1) + (size_t)HG * kKT + 3 * HG);
  if (lds > 160 * 1024) return (int)hipErrorInvalidValue;
  if (dt == 0) {
    auto k = latent_attn_rows_kernel<uint16_t, uint16_t>;
    if (lds > 48 * 1024) hipFuncSetAttribute((const void*)k, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    hipLaunchKernelGGL(k, dim3(n_rows), dim3(256), lds, s, qa, (const uint16_t*)cache, bt, maxb, row_seg, seg_row0,
                       seg_pos0, gate, ldg, (uint16_t*)out, row_base, H, R, BS, HG, scale, qst, qsh, qr, RP, ost, osh, window, sink);
  } else {
    auto k = latent_attn_rows_kernel<float, float>;
    if (lds > 48 * 1024) hipFuncSetAttribute((const void*)k, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    hipLaunchKernelGGL(k, dim3(n_rows), dim3(256), lds, s, qa, (const float*)cache, bt, maxb, row_seg, seg_row0,
                       seg_pos0, gate, ldg, (float*)out, row_base, H, R, BS, HG, scale, qst, qsh, qr, RP, ost, osh, window, sink);
  }
  return (int)hipGetLastError();
}

namespace k8s {

// ---------------------------------------------------------------------------
// MFMA form (bf16): v_mfma_f32_16x16x32_bf16, one wave per work item, no LDS.
//
// The latents are cached twice: c [pages][BS][R] (a key's R numbers contiguous:
// the QK^T operand) and ct [pages][R][BS] (8 consecutive keys of one latent
// column contiguous: the PV operand), as the K / transposed-V pages of the
// head-wise attention kernels.  A wave owns MT tiles of 16 query rows; a tile is
// TPM consecutive tokens x HC heads (HC = min(H, 16), TPM = 16 / HC), so all its
// rows read the same keys.  Keys go in chunks of 32 (never across a page:
// BS % 32 == 0).  Swapped QK^T (S^T = C Q^T): a lane owns ONE query row
// (lane & 15) and 8 of its key scores; MFMA row rho of key tile t holds key
// 8 (rho >> 2) + 4 t + (rho & 3), so lane quarter h ends with keys 8h .. 8h + 7,
// the k-slots of the PV operand: P moves from accumulator to operand in place.
//
// Items ([n][4] int32: segment, first row, tokens, position of the first row's
// token) are made on the host from the step's segments.  SPLIT (decode rows):
// grid.y partitions of `part` keys write unnormalised partials which
// latent_reduce merges -- the partition borders depend on the key index only,
// never on the batch (with a window a row's partitions start at the one its first
// visible key lies in).  Otherwise (prompt portions) a wave walks every key its
// rows see and writes the gated, normalised output.
//
// NP: 32-number chunks of the cache row behind the latent (a score-only key part): row width R + 32 NP.
constexpr float kLog2e = 1.4426950408889634f;

struct LatArgs {
  const uint16_t* qa;     // element (t, h, c) at t * qst + h * qsh + c
  long qst, qsh;
  const uint16_t* qr;     // [T][H][32 NP]
  const uint16_t* c;      // [pages][BS][R + 32 NP]
  const uint16_t* ct;     // [pages][R][BS]
  const int* bt;
  int maxb;
  const int* items;
  int n_items;
  const float* gate;      // or null
  int ldg;
  const float* sink;      // [H] or null
  int window;             // 0: every key up to the row's own position
  uint16_t* out;          // element (t, h, c) at t * ost + h * osh + c
  long ost, osh;
  float* part_o;          // [T][H][n_parts][R]
  float* part_ml;         // [T][H][n_parts][2]
  int n_parts, part;
  int H, HC, TPM, BS;
  float scale_log2;
};

__device__ __forceinline__ bf16x8 ld16(const uint16_t* p) { return *reinterpret_cast<const bf16x8*>(p); }

// One tile of 16 query rows meets 32 keys (scores s[2], keys kb + 8 h + 4 t + i): online softmax in log2 units.
// The weights go to pf (the PV product's operand); the accumulator o is rescaled only where a maximum moved.
template <int ND>
__device__ __forceinline__ void lat_softmax(const f32x4 (&s)[2], float scale_log2, bool open, int kb, int h, int lo,
                                            int limit, float& m, float& l, f32x4 (&o)[ND], bf16x8& pf) {
  float p[8];
#pragma unroll
  for (int t = 0; t < 2; ++t)
#pragma unroll
    for (int i = 0; i < 4; ++i) p[4 * t + i] = s[t][i] * scale_log2;
  if (!open) {                                             // (a wave-uniform branch)
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      const int key = kb + 8 * h + j;
      p[j] = key < limit && key >= lo ? p[j] : -INFINITY;
    }
  }
  float cmax = p[0];
#pragma unroll
  for (int j = 1; j < 8; ++j) cmax = fmaxf(cmax, p[j]);
  cmax = fmaxf(cmax, __shfl_xor(cmax, 16, 64));
  cmax = fmaxf(cmax, __shfl_xor(cmax, 32, 64));
  const bool grow = cmax > m;
  const float mn = grow ? cmax : m, ms = mn == -INFINITY ? 0.f : mn;    // -inf: a row that has seen no key yet
  float psum = 0.f;
#pragma unroll
  for (int j = 0; j < 8; ++j) {
    const float e = __builtin_amdgcn_exp2f(p[j] - ms);
    psum += e;
    pf[j] = (__bf16)e;
  }
  if (__any(grow)) {
    const float alpha = __builtin_amdgcn_exp2f(m - ms);
    l *= alpha;
    m = mn;
    float ar[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) ar[i] = __shfl(alpha, 4 * h + i, 64);
#pragma unroll
    for (int dt = 0; dt < ND; ++dt)
#pragma unroll
      for (int i = 0; i < 4; ++i) o[dt][i] *= ar[i];
  }
  l += psum;
}

template <int NR, int NP, int MT, bool SPLIT>
__global__ void __launch_bounds__(256) latent_attn_mfma_kernel(LatArgs a) {
  constexpr int R = NR * 32, ND = R / 16, NC = NR + NP, RW = R + 32 * NP;
  const int lane = threadIdx.x & 63, r = lane & 15, h = lane >> 4;
  // workgroups go round-robin over the 8 XCDs, each with its own L2: give every XCD a contiguous
  // range of items (neighbouring token groups of the same sequences read the same latent pages)
  const int per = gridDim.x >> 3;
  const int blk = (gridDim.x & 7) == 0 ? (blockIdx.x & 7) * per + (blockIdx.x >> 3) : blockIdx.x;
  const int item = blk * 4 + (threadIdx.x >> 6);
  if (item >= a.n_items) return;
  const int sg = a.items[item * 4], row0 = a.items[item * 4 + 1], ntok = a.items[item * 4 + 2],
            pos0 = a.items[item * 4 + 3];
  const int hc = blockIdx.z;
  int k_begin = a.window > 0 ? max(0, pos0 - a.window + 1) : 0, k_end = pos0 + ntok;
  if constexpr (SPLIT) {
    const int p0 = (k_begin / a.part + blockIdx.y) * a.part;
    k_begin = max(k_begin, p0);
    k_end = min(k_end, p0 + a.part);
    if (k_begin >= k_end) return;
  }
  // this lane's query row in every tile
  const int tl = r / a.HC, hl = r - tl * a.HC, head = hc * a.HC + hl;
  bf16x8 qf[MT][NC];
  int limit[MT], lo[MT];
  f32x4 o[MT][ND];
  float m[MT], l[MT];
#pragma unroll
  for (int mt = 0; mt < MT; ++mt) {
    const int ti = mt * a.TPM + tl;
    const bool valid = tl < a.TPM && ti < ntok && head < a.H;
    limit[mt] = valid ? min(pos0 + ti + 1, k_end) : 0;
    lo[mt] = max(k_begin, a.window > 0 ? pos0 + ti - a.window + 1 : 0);
    const size_t rq = row0 + (valid ? ti : 0), hq = valid ? head : 0;
#pragma unroll
    for (int cc = 0; cc < NC; ++cc) {
      qf[mt][cc] = ld16(cc < NR ? a.qa + rq * a.qst + hq * a.qsh + 32 * cc + 8 * h
                                : a.qr + (rq * a.H + hq) * (32 * NP) + 32 * (cc - NR) + 8 * h);
      if (!valid)
#pragma unroll
        for (int j = 0; j < 8; ++j) qf[mt][cc][j] = (__bf16)0.f;
    }
#pragma unroll
    for (int dt = 0; dt < ND; ++dt) o[mt][dt] = f32x4{0.f, 0.f, 0.f, 0.f};
    m[mt] = (!SPLIT && a.sink && valid) ? a.sink[head] * kLog2e : -INFINITY;
    l[mt] = 0.f;
  }
  const int* pages = a.bt + (size_t)sg * a.maxb;
  for (int kb = k_begin & ~31; kb < k_end; kb += 32) {
    const int page = pages[kb / a.BS], off = kb % a.BS;
    const uint16_t* cp = a.c + (size_t)page * a.BS * RW;
    const uint16_t* tp = a.ct + (size_t)page * R * a.BS;
    bf16x8 kf[2][NC];
#pragma unroll
    for (int t = 0; t < 2; ++t) {
      const int key = off + 8 * (r >> 2) + 4 * t + (r & 3);
#pragma unroll
      for (int cc = 0; cc < NC; ++cc) kf[t][cc] = ld16(cp + (size_t)key * RW + 32 * cc + 8 * h);
    }
    const bool open = kb >= k_begin && kb + 32 <= k_end && kb + 31 <= pos0 &&
                      (a.window <= 0 || kb >= pos0 + ntok - a.window);
    bf16x8 pf[MT];
#pragma unroll
    for (int mt = 0; mt < MT; ++mt) {
      f32x4 s[2];
#pragma unroll
      for (int t = 0; t < 2; ++t) {
        s[t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int cc = 0; cc < NC; ++cc)
          s[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[t][cc], qf[mt][cc], s[t], 0, 0, 0);
      }
      lat_softmax<ND>(s, a.scale_log2, open, kb, h, lo[mt], limit[mt], m[mt], l[mt], o[mt], pf[mt]);
    }
#pragma unroll
    for (int dt = 0; dt < ND; ++dt) {
      const bf16x8 vf = ld16(tp + (size_t)(16 * dt + r) * a.BS + off + 8 * h);
#pragma unroll
      for (int mt = 0; mt < MT; ++mt) o[mt][dt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(pf[mt], vf, o[mt][dt], 0, 0, 0);
    }
  }
#pragma unroll
  for (int mt = 0; mt < MT; ++mt) {
    float lt = l[mt];
    lt += __shfl_xor(lt, 16, 64);
    lt += __shfl_xor(lt, 32, 64);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int q = 4 * h + i;                       // the query row of accumulator element i
      const int qtl = q / a.HC, qhl = q - qtl * a.HC, qhead = hc * a.HC + qhl, ti = mt * a.TPM + qtl;
      const float lq = __shfl(lt, q, 64), mq = __shfl(m[mt], q, 64);
      if (!(qtl < a.TPM && ti < ntok && qhead < a.H)) continue;
      const size_t rh = (size_t)(row0 + ti) * a.H + qhead;
      if constexpr (SPLIT) {
        const size_t pi = rh * a.n_parts + blockIdx.y;
#pragma unroll
        for (int dt = 0; dt < ND; ++dt) a.part_o[pi * R + 16 * dt + r] = o[mt][dt][i];
        if (r == 0) {
          a.part_ml[pi * 2] = mq;
          a.part_ml[pi * 2 + 1] = lq;
        }
      } else {
        const float g = a.gate ? 1.f / (1.f + expf(-a.gate[(size_t)(row0 + ti) * a.ldg + qhead])) : 1.f;
        const float ls = a.sink ? lq + __builtin_amdgcn_exp2f(a.sink[qhead] * kLog2e - mq) : lq;
        const float sc = ls > 0.f ? g / ls : 0.f;
        uint16_t* op = a.out + (size_t)(row0 + ti) * a.ost + (size_t)qhead * a.osh + r;
#pragma unroll
        for (int dt = 0; dt < ND; ++dt) op[16 * dt] = f2bf(o[mt][dt][i] * sc);
      }
    }
  }
}

// Prompt portions: the four waves of a workgroup own four consecutive items of ONE
// segment (the host pads every segment's items to a multiple of four with empty
// ones), so they read the same keys.  A chunk's operand fragments do not depend on
// the item: kf[t][cc] and vf[dt] are loaded from global memory once per workgroup
// (a quarter by each wave), parked in LDS in fragment order -- slot f holds the 64
// lanes' 16 bytes, so writes and reads are conflict-free -- and read back by all
// four waves.  Two buffers: chunk i + 1 is fetched into registers while chunk i
// is computed, and written after it; one barrier per chunk.
template <int NR, int NP, int MT, int OCC>
__global__ void __launch_bounds__(256, OCC) latent_attn_mfma_lds_kernel(LatArgs a) {
  constexpr int R = NR * 32, ND = R / 16, NC = NR + NP, RW = R + 32 * NP, NF = 2 * NC + ND, NFW = (NF + 3) / 4;
  extern __shared__ __attribute__((aligned(16))) unsigned char lds_raw[];
  bf16x8* frag = reinterpret_cast<bf16x8*>(lds_raw);          // [2][NF][64]
  __shared__ int kend_s[4], kbeg_s[4];
  const int lane = threadIdx.x & 63, wv = threadIdx.x >> 6, r = lane & 15, h = lane >> 4;
  // ... and the LAST items of the range first: they see the most keys, so the short ones fill the tail
  const int per = gridDim.x >> 3;
  const int blk = (gridDim.x & 7) == 0 ? (blockIdx.x & 7) * per + (per - 1 - (blockIdx.x >> 3))
                                       : gridDim.x - 1 - blockIdx.x;
  const int item0 = blk * 4;
  if (item0 >= a.n_items) return;                              // whole workgroup
  const int item = item0 + wv;
  const int sg = a.items[item0 * 4];
  const int row0 = a.items[item * 4 + 1], ntok = a.items[item * 4 + 2], pos0 = a.items[item * 4 + 3];
  const int hc = blockIdx.z;
  if (lane == 0) {
    kend_s[wv] = ntok > 0 ? pos0 + ntok : 0;
    kbeg_s[wv] = ntok > 0 ? (a.window > 0 ? max(0, pos0 - a.window + 1) : 0) : 0x7fffffff;
  }
  __syncthreads();
  const int k_end = max(max(kend_s[0], kend_s[1]), max(kend_s[2], kend_s[3]));
  const int k_beg = min(min(kbeg_s[0], kbeg_s[1]), min(kbeg_s[2], kbeg_s[3])) & ~31;
  const int tl = r / a.HC, hl = r - tl * a.HC, head = hc * a.HC + hl;
  bf16x8 qf[MT][NC];
  int limit[MT], lo[MT];
  f32x4 o[MT][ND];
  float m[MT], l[MT];
#pragma unroll
  for (int mt = 0; mt < MT; ++mt) {
    const int ti = mt * a.TPM + tl;
    const bool valid = tl < a.TPM && ti < ntok && head < a.H;
    limit[mt] = valid ? pos0 + ti + 1 : 0;
    lo[mt] = a.window > 0 ? pos0 + ti - a.window + 1 : 0;
    const size_t rq = row0 + (valid ? ti : 0), hq = valid ? head : 0;
#pragma unroll
    for (int cc = 0; cc < NC; ++cc) {
      qf[mt][cc] = ld16(cc < NR ? a.qa + rq * a.qst + hq * a.qsh + 32 * cc + 8 * h
                                : a.qr + (rq * a.H + hq) * (32 * NP) + 32 * (cc - NR) + 8 * h);
      if (!valid)
#pragma unroll
        for (int j = 0; j < 8; ++j) qf[mt][cc][j] = (__bf16)0.f;
    }
#pragma unroll
    for (int dt = 0; dt < ND; ++dt) o[mt][dt] = f32x4{0.f, 0.f, 0.f, 0.f};
    m[mt] = (a.sink && valid) ? a.sink[head] * kLog2e : -INFINITY;
    l[mt] = 0.f;
  }
  const int* pages = a.bt + (size_t)sg * a.maxb;
  // this wave's share of a chunk's fragments: f = wv + 4 i
  bf16x8 pre[NFW];
  auto fetch = [&](int kb) {
    const int page = pages[kb / a.BS], off = kb % a.BS;
    const uint16_t* cp = a.c + (size_t)page * a.BS * RW;
    const uint16_t* tp = a.ct + (size_t)page * R * a.BS;
#pragma unroll
    for (int i = 0; i < NFW; ++i) {
      const int f = wv + 4 * i;
      if (f < 2 * NC) {
        const int t = f / NC, cc = f - t * NC;
        const int key = off + 8 * (r >> 2) + 4 * t + (r & 3);
        pre[i] = ld16(cp + (size_t)key * RW + 32 * cc + 8 * h);
      } else if (NF % 4 == 0 || f < NF) {
        const int dt = f - 2 * NC;
        pre[i] = ld16(tp + (size_t)(16 * dt + r) * a.BS + off + 8 * h);
      }
    }
  };
  auto park = [&](int buf) {
#pragma unroll
    for (int i = 0; i < NFW; ++i)
      if (NF % 4 == 0 || wv + 4 * i < NF) frag[((size_t)buf * NF + wv + 4 * i) * 64 + lane] = pre[i];
  };
  if (k_beg < k_end) {
    fetch(k_beg);
    park(0);
  }
  int buf = 0;
  for (int kb = k_beg; kb < k_end; kb += 32, buf ^= 1) {
    __syncthreads();
    const bool more = kb + 32 < k_end;
    if (more) fetch(kb + 32);
    const bf16x8* fb = frag + (size_t)buf * NF * 64 + lane;
    f32x4 s[MT][2];
#pragma unroll
    for (int t = 0; t < 2; ++t) {
#pragma unroll
      for (int mt = 0; mt < MT; ++mt) s[mt][t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int cc = 0; cc < NC; ++cc) {
        const bf16x8 kf = fb[(t * NC + cc) * 64];
#pragma unroll
        for (int mt = 0; mt < MT; ++mt)
          s[mt][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[mt][cc], s[mt][t], 0, 0, 0);
      }
    }
    const bool open = kb + 31 <= pos0 && (a.window <= 0 || kb >= pos0 + ntok - a.window);
    bf16x8 pf[MT];
#pragma unroll
    for (int mt = 0; mt < MT; ++mt)
      lat_softmax<ND>(s[mt], a.scale_log2, open, kb, h, lo[mt], limit[mt], m[mt], l[mt], o[mt], pf[mt]);
#pragma unroll
    for (int dt = 0; dt < ND; ++dt) {
      const bf16x8 vf = fb[(2 * NC + dt) * 64];
#pragma unroll
      for (int mt = 0; mt < MT; ++mt) o[mt][dt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(pf[mt], vf, o[mt][dt], 0, 0, 0);
    }
    if (more) park(buf ^ 1);
  }
#pragma unroll
  for (int mt = 0; mt < MT; ++mt) {
    float lt = l[mt];
    lt += __shfl_xor(lt, 16, 64);
    lt += __shfl_xor(lt, 32, 64);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int q = 4 * h + i;
      const int qtl = q / a.HC, qhl = q - qtl * a.HC, qhead = hc * a.HC + qhl, ti = mt * a.TPM + qtl;
      const float lq = __shfl(lt, q, 64), mq = __shfl(m[mt], q, 64);
      if (!(qtl < a.TPM && ti < ntok && qhead < a.H)) continue;
      const float g = a.gate ? 1.f / (1.f + expf(-a.gate[(size_t)(row0 + ti) * a.ldg + qhead])) : 1.f;
      const float ls = a.sink ? lq + __builtin_amdgcn_exp2f(a.sink[qhead] * kLog2e - mq) : lq;
      const float sc = ls > 0.f ? g / ls : 0.f;
      uint16_t* op = a.out + (size_t)(row0 + ti) * a.ost + (size_t)qhead * a.osh + r;
#pragma unroll
      for (int dt = 0; dt < ND; ++dt) op[16 * dt] = f2bf(o[mt][dt][i] * sc);
    }
  }
}

// Merge of the key partitions of decode rows: one workgroup per (row, head).
// A row at position p has the partitions from the one its first visible key lies in to p / part.
__global__ void __launch_bounds__(128) latent_reduce_kernel(const float* __restrict__ part_o,
                                                            const float* __restrict__ part_ml,
                                                            const int* __restrict__ positions,
                                                            const float* __restrict__ gate, int ldg,
                                                            uint16_t* __restrict__ out, int H, int R, int n_parts,
                                                            int part, long ost, long osh, int window,
                                                            const float* __restrict__ sink) {
  const int row = blockIdx.x / H, head = blockIdx.x - row * H;
  const size_t rh = (size_t)row * H + head;
  const int pos = positions[row], lo = window > 0 ? max(0, pos - window + 1) : 0;
  const int np = min(n_parts, pos / part - lo / part + 1);
  const float sk = sink ? sink[head] * kLog2e : -INFINITY;
  float mx = sk;
  for (int p = 0; p < np; ++p) mx = fmaxf(mx, part_ml[(rh * n_parts + p) * 2]);
  float lsum = sink ? exp2f(sk - mx) : 0.f;
  for (int p = 0; p < np; ++p) lsum += exp2f(part_ml[(rh * n_parts + p) * 2] - mx) * part_ml[(rh * n_parts + p) * 2 + 1];
  const float g = gate ? 1.f / (1.f + expf(-gate[(size_t)row * ldg + head])) : 1.f;
  for (int c = threadIdx.x; c < R; c += 128) {
    float acc = 0.f;
    for (int p = 0; p < np; ++p)
      acc = fmaf(exp2f(part_ml[(rh * n_parts + p) * 2] - mx), part_o[(rh * n_parts + p) * R + c], acc);
    out[row * ost + head * osh + c] = f2bf(acc / lsum * g);
  }
}

template <int NR, int NP>
static int launch_lat_np(const LatArgs& a, int split, int mt2, int n_head_chunks, hipStream_t s) {
  int nblk = (a.n_items + 3) / 4;
  if (nblk > 8) nblk = (nblk + 7) & ~7;   // a multiple of the XCD count (the kernels' item remap)
  const dim3 grid(nblk, split ? a.n_parts : 1, n_head_chunks);
  if (split) {
    hipLaunchKernelGGL((latent_attn_mfma_kernel<NR, NP, 1, true>), grid, dim3(256), 0, s, a);
    return (int)hipGetLastError();
  }
  if (a.n_items % 4) return (int)hipErrorInvalidValue;   // prompt items come in fours per segment
  constexpr size_t lds = 2 * (size_t)(4 * NR + 2 * NP) * 64 * 16;  // two buffers of 2 (NR + NP) + R / 16 KiB
  // tiles per wave and waves per SIMD by register need: two tiles while two waves still fit a SIMD
  // (R <= 128), one tile and two waves at R = 192 / 256, one and one above
  constexpr int MT = NR <= 4 ? 2 : 1, OCC = NR <= 8 ? 2 : 1;
  auto k = latent_attn_mfma_lds_kernel<NR, NP, MT, OCC>;
  if (lds > 48 * 1024 && hipFuncSetAttribute((const void*)k, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds))
    return (int)hipGetLastError();
  hipLaunchKernelGGL(k, grid, dim3(256), lds, s, a);
  return (int)hipGetLastError();
}

template <int NR>
static int launch_lat(const LatArgs& a, int np, int split, int mt2, int n_head_chunks, hipStream_t s) {
  switch (np) {
    case 0: return launch_lat_np<NR, 0>(a, split, mt2, n_head_chunks, s);
    case 1: return launch_lat_np<NR, 1>(a, split, mt2, n_head_chunks, s);
    case 2: return launch_lat_np<NR, 2>(a, split, mt2, n_head_chunks, s);
    default: return (int)hipErrorInvalidValue;
  }
}

}  // namespace k8s

// 0: the MFMA kernels do not take latent rank R; else the tiles per wave for prompt portions (2 up to R = 128).
// RP: the score-only numbers of a cache row behind the latent (a multiple of 32 up to 64).
K8S_API int k8s_latent_attn_mfma_ok(int R, int RP) {
  if (RP != 0 && RP != 32 && RP != 64) return 0;
  switch (R) {
    case 32: case 64: case 96: case 128: return 2;
    case 192: case 256: case 384: case 512: return 1;
    default: return 0;
  }
}

// split = 1: decode rows (items of one token), partials + merge into out; `positions` [T] are the
// rows' positions and n_rows the number of decode rows (the first rows of the step).
// split = 0: prompt portions, items of up to tiles * (16 / min(H, 16)) tokens.
K8S_API int k8s_latent_attn_mfma(const void* qa, const void* c, const void* ct, const int* bt, int maxb,
                                 const int* items, int n_items, const float* gate, int ldg, void* out,
                                 float* part_o, float* part_ml, int n_parts, int part, const int* positions,
                                 int n_rows, int H, int R, int BS, float scale, int split, int tiles,
                                 hipStream_t s, long qst, long qsh, const void* qr, int RP, long ost, long osh,
                                 int window, const float* sink) {
  if (n_items <= 0) return 0;
  if (!k8s_latent_attn_mfma_ok(R, RP) || BS % 32 || H <= 0 || (split && part % 32) || (RP && !qr) || window < 0 ||
      qst % 8 || qsh % 8)
    return (int)hipErrorInvalidValue;
  k8s::LatArgs a;
  a.qst = qst; a.qsh = qsh; a.qr = (const uint16_t*)qr; a.ost = ost; a.osh = osh; a.window = window; a.sink = sink;
  a.qa = (const uint16_t*)qa; a.c = (const uint16_t*)c; a.ct = (const uint16_t*)ct; a.bt = bt; a.maxb = maxb;
  a.items = items; a.n_items = n_items; a.gate = gate; a.ldg = ldg; a.out = (uint16_t*)out;
  a.part_o = part_o; a.part_ml = part_ml; a.n_parts = n_parts; a.part = part;
  a.H = H; a.HC = H < 16 ? H : 16; a.TPM = 16 / a.HC; a.BS = BS; a.scale_log2 = scale * k8s::kLog2e;
  const int nhc = (H + a.HC - 1) / a.HC, mt2 = (!split && tiles == 2);
  int rc;
  switch (R / 32) {
    case 1: rc = k8s::launch_lat<1>(a, RP / 32, split, mt2, nhc, s); break;
    case 2: rc = k8s::launch_lat<2>(a, RP / 32, split, mt2, nhc, s); break;
    case 3: rc = k8s::launch_lat<3>(a, RP / 32, split, mt2, nhc, s); break;
    case 4: rc = k8s::launch_lat<4>(a, RP / 32, split, mt2, nhc, s); break;
    case 6: rc = k8s::launch_lat<6>(a, RP / 32, split, mt2, nhc, s); break;
    case 8: rc = k8s::launch_lat<8>(a, RP / 32, split, mt2, nhc, s); break;
    case 12: rc = k8s::launch_lat<12>(a, RP / 32, split, mt2, nhc, s); break;
    case 16: rc = k8s::launch_lat<16>(a, RP / 32, split, mt2, nhc, s); break;
    default: return (int)hipErrorInvalidValue;
  }
  if (rc || !split) return rc;
  hipLaunchKernelGGL(k8s::latent_reduce_kernel, dim3(n_rows * H), dim3(128), 0, s, part_o, part_ml, positions, gate, ldg,
                     (uint16_t*)out, H, R, n_parts, part, ost, osh, window, sink);
  return (int)hipGetLastError();
}
