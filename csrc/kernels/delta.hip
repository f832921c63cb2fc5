// Gated delta rule (gfx950).  Per head a state S [d, vd] fp32 that a scalar decay shrinks and a rank-one step corrects:
//   g_t = exp(-exp(A_log_h) softplus(a_t + dt_bias_h)),  beta_t = sigmoid(b_t),  k, q unit vectors (q times d^-1/2)
//   S <- g_t S;  u_t = beta_t (v_t - S^T k_t);  S <- S + k_t u_t^T;  o_t = S^T q_t
// Portions run in chunks of DC = 64 tokens.  With L_t the sum of log g up to token t of the chunk, S_0 the state at its
// start and
//   A_ts = beta_t e^(L_t - L_s) k_t.k_s  (s < t),   T = (I + A)^-1,   M_ts = e^(L_t - L_s) q_t.k_s  (s <= t)
// the recurrence unrolls to
//   U = T (beta v - beta e^L K S_0),   o_t = e^(L_t) S_0^T q_t + (M U)_t,   S_end = e^(L_63) S_0 + sum_t e^(L_63 - L_t) k_t u_t^T
// so that all work but S_0 -> S_end is independent between chunks, and between the columns of S everywhere:
//   delta_prep_kernel   per (head, chunk): norms, decays, T and M, and the operands of the scan in matrix-core lane order;
//   delta_scan_kernel   per (sequence, head, 16 columns of S): walks the chunks, S in registers;
//   delta_step_kernel   one token per sequence (decode), the gated RMS norm behind it included.
// Everything is fp32.  q, k and v come as projected and convolved (bf16 or fp32, dt: 0 = bf16, 1 = fp32); their unit norms
// are scalars per token that join beside the products.  For bf16, products of q / k entries with each other are exact
// on the bf16 matrix cores (fp32 sums); their products with an fp32 matrix take it as the sum of three bf16 parts (8 + 8 +
// 8 mantissa bits), three matrix-core steps.  The other products, and all of them for fp32, are fp32 matrix-core steps.
// A sequence whose first token of the step sits at position 0 starts from zeros instead of its slot's contents.
#include "common.h"

GRAG_ERR_UNIT(delta)

namespace grag {

constexpr int DC = 64;            // tokens per chunk
constexpr int DMAX = 256;         // head sizes at most
constexpr int HB_FLOATS = 5440;   // per (chunk, head): T 10 x 256 | M 10 x 256 | 4 x 64 scalars | e^(L_63), padding

template <typename T> __device__ __forceinline__ float ldd(const T* p);
template <> __device__ __forceinline__ float ldd<bf16>(const bf16* p) { return (float)*p; }
template <> __device__ __forceinline__ float ldd<float>(const float* p) { return *p; }
template <typename T> __device__ __forceinline__ void std_(T* p, float v);
template <> __device__ __forceinline__ void std_<bf16>(bf16* p, float v) { *p = (bf16)v; }
template <> __device__ __forceinline__ void std_<float>(float* p, float v) { *p = v; }

__device__ __forceinline__ float softplus_d(float x) { return x > 20.f ? x : log1pf(expf(x)); }
__device__ __forceinline__ float sigmoid_d(float x) { return 1.f / (1.f + expf(-x)); }
__device__ __forceinline__ float log_decay(float a, float dtb, float alog) { return -expf(alog) * softplus_d(a + dtb); }

// ------------------------------------------------------------------------------------------------ matrix-core operands
// Lane l of a wave: ql = l % 16, quad = l / 16.  A 16 x 16 fp32 block in result order: lane holds rows 4 quad + i (i < 4)
// of column ql.  As the order of a sum is free, the same four numbers are the lane's share of the right operand of a
// product over the block's 16 rows, if the left operand's lane holds row ql at the columns 4 quad + i.
// A left operand for 32 columns ("frag"): row ql at columns 4 quad + 0..3 and 16 + 4 quad + 0..3.
template <typename T> struct Frag;
template <> struct Frag<bf16> {
  bf16x8_t v;
  __device__ __forceinline__ void load(const bf16* p) { v = *reinterpret_cast<const bf16x8_t*>(p); }
};
template <> struct Frag<float> {
  f32x4_t v[2];
  __device__ __forceinline__ void load(const float* p) {
    v[0] = *reinterpret_cast<const f32x4_t*>(p);
    v[1] = *reinterpret_cast<const f32x4_t*>(p + 4);
  }
};

__device__ __forceinline__ f32x4_t mm16(f32x4_t a, f32x4_t b, f32x4_t acc) {  // fp32, 16 columns
#pragma unroll
  for (int i = 0; i < 4; ++i) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a[i], b[i], acc, 0, 0, 0);
  return acc;
}

// The fp32 right operand (32 rows: two result-order blocks) of a product with a T left operand, in LDS: for bf16 the
// three parts, each lane's 8 numbers per part; for fp32 the numbers themselves.
template <typename T> struct Right;
template <> struct Right<bf16> {
  static constexpr int PLANES = 3;
  bf16x8_t p[3];
  __device__ __forceinline__ void load(const bf16* s, int lane) {
#pragma unroll
    for (int j = 0; j < 3; ++j) p[j] = *reinterpret_cast<const bf16x8_t*>(s + (j * 64 + lane) * 8);
  }
  static __device__ __forceinline__ void store(bf16* s, int lane, int half, f32x4_t x) {
    bf16x4_t h, m, l;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      h[i] = f2bits(x[i]);
      const float r = x[i] - bits2f(h[i]);
      m[i] = f2bits(r);
      l[i] = f2bits(r - bits2f(m[i]));
    }
    *reinterpret_cast<bf16x4_t*>(s + (0 * 64 + lane) * 8 + 4 * half) = h;
    *reinterpret_cast<bf16x4_t*>(s + (1 * 64 + lane) * 8 + 4 * half) = m;
    *reinterpret_cast<bf16x4_t*>(s + (2 * 64 + lane) * 8 + 4 * half) = l;
  }
};
template <> struct Right<float> {
  static constexpr int PLANES = 1;
  f32x4_t p[2];
  __device__ __forceinline__ void load(const float* s, int lane) {
    p[0] = *reinterpret_cast<const f32x4_t*>(s + lane * 8);
    p[1] = *reinterpret_cast<const f32x4_t*>(s + lane * 8 + 4);
  }
  static __device__ __forceinline__ void store(float* s, int lane, int half, f32x4_t x) {
    *reinterpret_cast<f32x4_t*>(s + lane * 8 + 4 * half) = x;
  }
};
__device__ __forceinline__ f32x4_t mm32(const Frag<bf16>& a, const Right<bf16>& b, f32x4_t acc) {
#pragma unroll
  for (int j = 2; j >= 0; --j) acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.v, b.p[j], acc, 0, 0, 0);
  return acc;
}
__device__ __forceinline__ f32x4_t mm32(const Frag<float>& a, const Right<float>& b, f32x4_t acc) {
  return mm16(a.v[1], b.p[1], mm16(a.v[0], b.p[0], acc));
}

// sum over groups of 4 neighbouring lanes, in every lane
__device__ __forceinline__ float sum4(float v) {
  v += __shfl_xor(v, 1, 64);
  v += __shfl_xor(v, 2, 64);
  return v;
}

// the scratch row of a sequence's first chunk (rows of unequal sequences never meet: a sequence that starts at token qa
// and has n tokens uses at most (qa + n) / DC - qa / DC + 1 of them)
__device__ __forceinline__ int chunk_row(int qa, int seq) { return qa / DC + seq; }

// ------------------------------------------------------------------------------------------------ operands of the scan
// grid (H, max chunks, nseq), 256 threads.  wk [nchunks][G] blocks of 3 DC dp T's: K frags [4][ND][64][8], Q frags (the
// same), K^T frags [2 ND][2][64][8] (dp = 32 ND: d rounded up, zeros behind d); wh [nchunks][H] blocks of HB_FLOATS.
// Lower block (i, j <= i) of a 64 x 64 triangle has number i (i + 1) / 2 + j.
template <typename T>
__global__ void __launch_bounds__(256)
delta_prep_kernel(const T* __restrict__ xc, int C, const T* __restrict__ proj, int ld, int boff, int aoff,
                  const float* __restrict__ a_log, const float* __restrict__ dt_bias, const int* __restrict__ q_start,
                  int H, int G, int d, int vec, T* __restrict__ wk, float* __restrict__ wh, int nchunks) {
  extern __shared__ __attribute__((aligned(16))) unsigned char dsm[];
  const int seq = blockIdx.z, c = blockIdx.y, h = blockIdx.x, R = H / G, gk = h / R;
  const int qa = q_start[seq], qlen = q_start[seq + 1] - qa;
  if (c * DC >= qlen) return;
  const int crow = chunk_row(qa, seq) + c;
  if (crow >= nchunks) return;
  const int nrow = min(DC, qlen - c * DC), r0 = qa + c * DC;
  const int ND = (d + 31) / 32, dp = 32 * ND, lk = dp + (sizeof(T) == 2 ? 8 : 4);
  T* Ks = reinterpret_cast<T*>(dsm);
  T* Qs = Ks + DC * lk;
  float* Ts = reinterpret_cast<float*>(dsm);  // [64][68], in the place of K and Q once they have been used
  float* Af = Ts + max(DC * 68, 2 * DC * lk * (int)sizeof(T) / 4);  // [10][64][4]
  float* rk = Af + 2560;                               // [64] each: 1 / |k|, d^-1/2 / |q|, L (two parts), beta
  float *rq = rk + DC, *lh = rq + DC, *ll = lh + DC, *be = ll + DC;
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, ql = lane & 15, quad = lane >> 4;
  {  // rows of K and Q, zeros behind d and behind the portion's end
    const int row = threadIdx.x >> 2, part = threadIdx.x & 3;
    const T* src = xc + (size_t)(r0 + (row < nrow ? row : 0)) * C + gk * d;
    float sk = 0.f, sq = 0.f;
    for (int k0 = part * 8; k0 < dp; k0 += 32) {
      T kv[8], qv[8];
      if (vec && row < nrow && k0 < d) {
        Frag<T> fk, fq;
        fq.load(src + k0);
        fk.load(src + G * d + k0);
        __builtin_memcpy(qv, &fq, sizeof(qv));
        __builtin_memcpy(kv, &fk, sizeof(kv));
      } else {
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          const bool ok = row < nrow && k0 + e < d;
          qv[e] = ok ? src[k0 + e] : (T)0.f;
          kv[e] = ok ? src[G * d + k0 + e] : (T)0.f;
        }
      }
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        sk = fmaf((float)kv[e], (float)kv[e], sk);
        sq = fmaf((float)qv[e], (float)qv[e], sq);
        Ks[row * lk + k0 + e] = kv[e];
        Qs[row * lk + k0 + e] = qv[e];
      }
    }
    sk = sum4(sk);
    sq = sum4(sq);
    if (part == 0) {
      rk[row] = 1.f / sqrtf(sk + 1e-6f);
      rq[row] = 1.f / sqrtf(sq + 1e-6f) / sqrtf((float)d);
    }
  }
  if (w == 0) {
    float lg = 0.f, bt = 0.f;
    if (lane < nrow) {
      const T* p = proj + (size_t)(r0 + lane) * ld;
      lg = log_decay(ldd(p + aoff + h), dt_bias[h], a_log[h]);
      bt = sigmoid_d(ldd(p + boff + h));
    }
    double s = lg;  // (the sums grow with the chunk, their differences need not: two floats keep them)
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const double u = __shfl_up(s, o, 64);
      if (lane >= o) s += u;
    }
    lh[lane] = (float)s;
    ll[lane] = (float)(s - (double)(float)s);
    be[lane] = bt;
  }
  __syncthreads();
  float* hb = wh + ((size_t)crow * H + h) * HB_FLOATS;
  if (h % R == 0) {  // the heads of a q / k head share its frags
    T* kb = wk + ((size_t)crow * G + gk) * 3 * DC * dp;
    T* qb = kb + DC * dp;
    T* tb = qb + DC * dp;
    for (int idx = threadIdx.x; idx < 4 * ND * 64; idx += 256) {
      const int l = idx & 63, kg = (idx >> 6) % ND, rb = (idx >> 6) / ND;
      const int o = (16 * rb + (l & 15)) * lk + 32 * kg + 4 * (l >> 4);
      T kv[8], qv[8];
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        const int oo = o + (e < 4 ? e : 12 + e);
        kv[e] = Ks[oo];
        qv[e] = Qs[oo];
      }
      __builtin_memcpy(__builtin_assume_aligned(kb + (size_t)idx * 8, 16), kv, sizeof(kv));
      __builtin_memcpy(__builtin_assume_aligned(qb + (size_t)idx * 8, 16), qv, sizeof(qv));
    }
    for (int idx = threadIdx.x; idx < 2 * ND * 2 * 64; idx += 256) {
      const int l = idx & 63, ks = (idx >> 6) & 1, rb = idx >> 7;
      T kv[8];
#pragma unroll
      for (int e = 0; e < 8; ++e)
        kv[e] = Ks[(32 * ks + 4 * (l >> 4) + (e < 4 ? e : 12 + e)) * lk + 16 * rb + (l & 15)];
      __builtin_memcpy(__builtin_assume_aligned(tb + (size_t)idx * 8, 16), kv, sizeof(kv));
    }
  }
  // the triangles A (into LDS) and M (into the scratch), transposed products: rows s, column t, which is the order a left
  // operand with row t wants
  for (int idx = w; idx < 20; idx += 4) {
    const int p = idx % 10, i = p < 1 ? 0 : p < 3 ? 1 : p < 6 ? 2 : 3, j = p - i * (i + 1) / 2;
    const bool isq = idx >= 10;
    const T* ap = Ks + (16 * j + ql) * lk;
    const T* bp = (isq ? Qs : Ks) + (16 * i + ql) * lk;
    f32x4_t acc = f32x4_t{0.f, 0.f, 0.f, 0.f};
    for (int kg = 0; kg < ND; ++kg) {
      if constexpr (sizeof(T) == 2) {
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf16x8_t*>(ap + 32 * kg + 8 * quad),
                                                      *reinterpret_cast<const bf16x8_t*>(bp + 32 * kg + 8 * quad), acc, 0,
                                                      0, 0);
      } else {
#pragma unroll
        for (int e = 0; e < 2; ++e)
          acc = mm16(*reinterpret_cast<const f32x4_t*>(ap + 32 * kg + 16 * e + 4 * quad),
                     *reinterpret_cast<const f32x4_t*>(bp + 32 * kg + 16 * e + 4 * quad), acc);
      }
    }
    const int t = 16 * i + ql;
    const float lt = lh[t], lt2 = ll[t], ft = isq ? rq[t] : be[t] * rk[t];
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int s = 16 * j + 4 * quad + r;
      const float e = expf(fminf((lt - lh[s]) + (lt2 - ll[s]), 0.f)) * ft * rk[s];
      acc[r] = (isq ? s <= t : s < t) ? acc[r] * e : 0.f;
    }
    float* dst = isq ? hb + 2560 + p * 256 : Af + p * 256;
    *reinterpret_cast<f32x4_t*>(dst + lane * 4) = acc;
  }
  if (w == 3) {
    const float lt = lh[lane] + ll[lane], el = expf(lt);
    const float ec = expf(fminf((lh[DC - 1] - lh[lane]) + (ll[DC - 1] - ll[lane]), 0.f));
    hb[5120 + lane] = be[lane] * el * rk[lane];
    hb[5120 + 64 + lane] = be[lane];
    hb[5120 + 128 + lane] = el * rq[lane];
    hb[5120 + 192 + lane] = ec * rk[lane];
    if (lane == DC - 1) hb[5120 + 256] = el;
  }
  __syncthreads();
  {  // inverse of the diagonal blocks, by substitution: lane ql forms column ql of block w
    const float* Ad = Af + (w * (w + 1) / 2 + w) * 256;
    float x[16];
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      float a = r == ql ? 1.f : 0.f;
#pragma unroll
      for (int s4 = 0; s4 < (r + 3) / 4; ++s4) {
        const f32x4_t v = *reinterpret_cast<const f32x4_t*>(Ad + (r + 16 * s4) * 4);
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (4 * s4 + e < r) a = fmaf(-v[e], x[4 * s4 + e], a);
      }
      x[r] = a;
    }
    if (quad == 0) {
#pragma unroll
      for (int r = 0; r < 16; ++r) Ts[(16 * w + r) * 68 + 16 * w + ql] = x[r];
    }
  }
  __syncthreads();
  {  // the blocks below: wave w walks block column w, T_i = -T_ii sum_(w <= k < i) A_ik T_k
    f32x4_t X[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      X[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
      if (i < w) continue;
      if (i == w) {
#pragma unroll
        for (int r = 0; r < 4; ++r) X[i][r] = Ts[(16 * i + 4 * quad + r) * 68 + 16 * w + ql];
        continue;
      }
      f32x4_t acc = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int k = 0; k < i; ++k)
        if (k >= w) acc = mm16(*reinterpret_cast<const f32x4_t*>(Af + (i * (i + 1) / 2 + k) * 256 + lane * 4), X[k], acc);
      X[i] = mm16(*reinterpret_cast<const f32x4_t*>(Ts + (16 * i + ql) * 68 + 16 * i + 4 * quad), -acc,
                  f32x4_t{0.f, 0.f, 0.f, 0.f});
#pragma unroll
      for (int r = 0; r < 4; ++r) Ts[(16 * i + 4 * quad + r) * 68 + 16 * w + ql] = X[i][r];
    }
  }
  __syncthreads();
  for (int idx = threadIdx.x; idx < 640; idx += 256) {
    const int l = idx & 63, p = idx >> 6, i = p < 1 ? 0 : p < 3 ? 1 : p < 6 ? 2 : 3, j = p - i * (i + 1) / 2;
    *reinterpret_cast<f32x4_t*>(hb + idx * 4) =
        *reinterpret_cast<const f32x4_t*>(Ts + (16 * i + (l & 15)) * 68 + 16 * j + 4 * (l >> 4));
  }
}

// ------------------------------------------------------------------------------------------------ scan over the chunks
// grid nseq * H * ceil(vd / 16) (the column tiles of a head beside each other, on one XCD), 256 threads.  Wave w has token
// block w of every chunk and rows 32 kg .. + 31 of the state's 16 columns for kg = w, w + 4.  NDM >= ND = ceil(d / 32).
template <typename T, int NDM>
__global__ void __launch_bounds__(256)
delta_scan_kernel(const T* __restrict__ xc, int C, float* __restrict__ state, const int* __restrict__ slots,
                  const int* __restrict__ q_start, const int* __restrict__ ctx_len, float* __restrict__ out, int H, int G,
                  int d, int vd, int nslots, const T* __restrict__ wk, const float* __restrict__ wh, int nchunks) {
  constexpr int NG = (NDM + 3) / 4, RS = Right<T>::PLANES * 512;
  __shared__ __attribute__((aligned(16))) T So[NDM * RS];  // S_0 as right operands
  __shared__ __attribute__((aligned(16))) T Co[2 * RS];    // e^(L_63 - L_t) / |k_t| u_t as right operands
  __shared__ __attribute__((aligned(16))) float Rl[4][256], Ul[4][256];
  const int ntile = (vd + 15) / 16;
  const int id = xcd_remap(blockIdx.x, gridDim.x);
  const int tile = id % ntile, h = (id / ntile) % H, seq = id / ntile / H;
  const int qa = q_start[seq], qlen = q_start[seq + 1] - qa;
  if (qlen <= 0) return;
  const int lane = threadIdx.x & 63, w = threadIdx.x >> 6, ql = lane & 15, quad = lane >> 4;
  const int ND = (d + 31) / 32, dp = 32 * ND, gk = h / (H / G), n = 16 * tile + ql;
  const bool n_ok = n < vd, fresh = ctx_len[seq] - qlen == 0;
  const int slot = slots[seq];
  const bool slot_ok = index_ok(slot, nslots, ERR_SAMPLER_SLOT);
  float* Sg = state + ((size_t)(slot_ok ? slot : 0) * H + h) * d * vd + n;
  const int crow = chunk_row(qa, seq), nch = (qlen + DC - 1) / DC;
  if (crow + nch > nchunks) return;
  f32x4_t S[NG][2];
#pragma unroll
  for (int g = 0; g < NG; ++g)
#pragma unroll
    for (int b = 0; b < 2; ++b) {
      const int kg = w + 4 * g;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int r = 32 * kg + 16 * b + 4 * quad + i;
        S[g][b][i] = !fresh && slot_ok && n_ok && r < d ? Sg[(size_t)r * vd] : 0.f;
      }
      if (kg < ND) Right<T>::store(So + kg * RS, lane, b, S[g][b]);
    }
  const size_t kstep = (size_t)G * 3 * DC * dp, hstep = (size_t)H * HB_FLOATS;
  const T* kb = wk + ((size_t)crow * G + gk) * 3 * DC * dp;
  const float* hb = wh + ((size_t)crow * H + h) * HB_FLOATS;
  const T* vp = xc + (size_t)(qa + 16 * w + 4 * quad) * C + 2 * G * d + h * vd + (n_ok ? n : 0);
  float* op = out + (size_t)(qa + 16 * w + 4 * quad) * (size_t)(H * vd) + h * vd + n;
  // operands of the chunk at hand; each set is fetched for the next chunk as soon as this one has used it
  Frag<T> kf[NDM], qf[NDM], tf[NG][2][2];
  f32x4_t Tf[4], Mf[4], sa, sb, sq, sc;
  T vv[4];
  float end;
  auto fetch_qk = [&](const T* kc, const float* hc, int left) {
#pragma unroll
    for (int k = 0; k < NDM; ++k)
      if (k < ND) {
        kf[k].load(kc + ((w * ND + k) * 64 + lane) * 8);
        qf[k].load(kc + DC * dp + ((w * ND + k) * 64 + lane) * 8);
      }
    sa = *reinterpret_cast<const f32x4_t*>(hc + 5120 + 16 * w + 4 * quad);
    sb = *reinterpret_cast<const f32x4_t*>(hc + 5120 + 64 + 16 * w + 4 * quad);
#pragma unroll
    for (int i = 0; i < 4; ++i) vv[i] = 16 * w + 4 * quad + i < left ? vp[(size_t)i * C] : (T)0.f;
  };
  auto fetch_t = [&](const float* hc) {
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (j <= w) Tf[j] = *reinterpret_cast<const f32x4_t*>(hc + (w * (w + 1) / 2 + j) * 256 + lane * 4);
    sc = *reinterpret_cast<const f32x4_t*>(hc + 5120 + 192 + 16 * w + 4 * quad);
  };
  auto fetch_m = [&](const T* kc, const float* hc) {
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (j <= w) Mf[j] = *reinterpret_cast<const f32x4_t*>(hc + 2560 + (w * (w + 1) / 2 + j) * 256 + lane * 4);
    sq = *reinterpret_cast<const f32x4_t*>(hc + 5120 + 128 + 16 * w + 4 * quad);
    end = hc[5120 + 256];
#pragma unroll
    for (int g = 0; g < NG; ++g)
      if (w + 4 * g < ND) {
#pragma unroll
        for (int b = 0; b < 2; ++b)
#pragma unroll
          for (int ks = 0; ks < 2; ++ks)
            tf[g][b][ks].load(kc + 2 * DC * dp + (((2 * (w + 4 * g) + b) * 2 + ks) * 64 + lane) * 8);
      }
  };
  fetch_qk(kb, hb, qlen);
  fetch_t(hb);
  fetch_m(kb, hb);
  const f32x4_t zero = f32x4_t{0.f, 0.f, 0.f, 0.f};
  for (int c = 0; c < nch; ++c) {
    const bool more = c + 1 < nch;
    const int left = qlen - c * DC;
    __syncthreads();
    // the start state seen by the chunk's keys and queries, and the right-hand side of the triangular system
    f32x4_t ks = zero, qs = zero;
#pragma unroll
    for (int k = 0; k < NDM; ++k)
      if (k < ND) {
        Right<T> b;
        b.load(So + k * RS, lane);
        ks = mm32(kf[k], b, ks);
        qs = mm32(qf[k], b, qs);
      }
    f32x4_t r;
#pragma unroll
    for (int i = 0; i < 4; ++i) r[i] = fmaf(sb[i], (float)vv[i], -sa[i] * ks[i]);
    *reinterpret_cast<f32x4_t*>(&Rl[w][lane * 4]) = r;
    vp += (size_t)DC * C;
    if (more) fetch_qk(kb + kstep, hb + hstep, left - DC);
    __syncthreads();
    f32x4_t u = zero;
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (j <= w) u = mm16(Tf[j], *reinterpret_cast<const f32x4_t*>(&Rl[j][lane * 4]), u);
    *reinterpret_cast<f32x4_t*>(&Ul[w][lane * 4]) = u;
    Right<T>::store(Co + (w >> 1) * RS, lane, w & 1, sc * u);
    if (more) fetch_t(hb + hstep);
    __syncthreads();
    f32x4_t o = sq * qs;
#pragma unroll
    for (int j = 0; j < 4; ++j)
      if (j <= w) o = mm16(Mf[j], *reinterpret_cast<const f32x4_t*>(&Ul[j][lane * 4]), o);
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (n_ok && 16 * w + 4 * quad + i < left) op[(size_t)i * (H * vd)] = o[i];
    op += (size_t)DC * (H * vd);
    Right<T> cu[2];
#pragma unroll
    for (int k = 0; k < 2; ++k) cu[k].load(Co + k * RS, lane);
#pragma unroll
    for (int g = 0; g < NG; ++g) {
      if (w + 4 * g >= ND) continue;
#pragma unroll
      for (int b = 0; b < 2; ++b) {
        S[g][b] = mm32(tf[g][b][1], cu[1], mm32(tf[g][b][0], cu[0], end * S[g][b]));
        Right<T>::store(So + (w + 4 * g) * RS, lane, b, S[g][b]);
      }
    }
    kb += kstep;
    hb += hstep;
    if (more) fetch_m(kb, hb);
  }
  if (!slot_ok || !n_ok) return;
#pragma unroll
  for (int g = 0; g < NG; ++g)
#pragma unroll
    for (int b = 0; b < 2; ++b)
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int r = 32 * (w + 4 * g) + 16 * b + 4 * quad + i;
        if (r < d) Sg[(size_t)r * vd] = S[g][b][i];
      }
}

// ------------------------------------------------------------------------------------------------ one token
// grid (H, nseq), up to NT threads: a thread holds V columns of the rows rg, rg + RG, ... (at most RPT of them) of its head's
// state, ncp = 2^n >= vd / V threads a row, RG = NT / ncp row groups.  The state is read once and written once; S^T k and
// S^T q are sums over the row groups.  Then y = o / rms(o) * w * silu(gate).
template <int V> __device__ __forceinline__ void ldV(const float* p, float (&v)[V]) {
  if constexpr (V == 4) {
    const f32x4_t t = *reinterpret_cast<const f32x4_t*>(p);
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = t[i];
  } else {
    v[0] = *p;
  }
}
template <int V> __device__ __forceinline__ void stV(float* p, const float (&v)[V]) {
  if constexpr (V == 4) *reinterpret_cast<f32x4_t*>(p) = f32x4_t{v[0], v[1], v[2], v[3]};
  else *p = v[0];
}

template <typename T, int V, int RPT, int NT>
__global__ void __launch_bounds__(NT)
delta_step_kernel(const T* __restrict__ xc, int C, const T* __restrict__ proj, int ld, int boff, int aoff, int goff,
                  const float* __restrict__ a_log, const float* __restrict__ dt_bias, const float* __restrict__ wn,
                  float eps, float* __restrict__ state, const int* __restrict__ slots, const int* __restrict__ q_start,
                  const int* __restrict__ ctx_len, T* __restrict__ y, int H, int G, int d, int vd, int nslots, int ncp) {
  __shared__ float ks[DMAX], qs[DMAX], gb[2], red[16];
  __shared__ __attribute__((aligned(16))) float part[2][16 * 256];  // [sums at hand][row group or wave][columns]
  const int h = blockIdx.x, seq = blockIdx.y;
  const int row = q_start[seq];
  if (q_start[seq + 1] <= row) return;
  const bool fresh = ctx_len[seq] == 1;
  const int slot = slots[seq];
  const bool slot_ok = index_ok(slot, nslots, ERR_SAMPLER_SLOT);
  float* Sg = state + ((size_t)(slot_ok ? slot : 0) * H + h) * d * vd;
  const int cp = threadIdx.x & (ncp - 1), rg = threadIdx.x / ncp, RG = blockDim.x / ncp, c0 = cp * V;
  const bool c_ok = c0 < vd;
  float S[RPT][V];
#pragma unroll
  for (int u = 0; u < RPT; ++u) {
#pragma unroll
    for (int i = 0; i < V; ++i) S[u][i] = 0.f;
    const int r = rg + RG * u;
    if (!fresh && slot_ok && c_ok && r < d) ldV<V>(Sg + (size_t)r * vd + c0, S[u]);
  }
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6, nw = blockDim.x >> 6;
  if (wid < 2) {  // wave 0: the key, wave 1: the query
    const T* src = xc + (size_t)row * C + (wid == 0 ? G * d : 0) + h / (H / G) * d;
    float v[DMAX / 64], ss = 0.f;
#pragma unroll
    for (int u = 0; u < DMAX / 64; ++u) {
      v[u] = lane + 64 * u < d ? ldd(src + lane + 64 * u) : 0.f;
      ss = fmaf(v[u], v[u], ss);
    }
    float r = 1.f / sqrtf(wave_sum(ss) + 1e-6f);
    if (wid == 1) r /= sqrtf((float)d);
#pragma unroll
    for (int u = 0; u < DMAX / 64; ++u)
      if (lane + 64 * u < d) (wid == 0 ? ks : qs)[lane + 64 * u] = v[u] * r;
  } else if (threadIdx.x == 128) {
    const T* p = proj + (size_t)row * ld;
    gb[0] = expf(log_decay(ldd(p + aoff + h), dt_bias[h], a_log[h]));
    gb[1] = sigmoid_d(ldd(p + boff + h));
  }
  float vv[V], gt[V];
#pragma unroll
  for (int i = 0; i < V; ++i) {
    vv[i] = c_ok ? ldd(xc + (size_t)row * C + 2 * G * d + h * vd + c0 + i) : 0.f;
    gt[i] = rg == 0 && c_ok ? ldd(proj + (size_t)row * ld + goff + h * vd + c0 + i) : 0.f;
  }
  // the sums over the row groups: lanes of a wave first, then the waves (or, for rows wider than a wave, the groups)
  const int npart = ncp < 64 ? nw : RG, mypart = ncp < 64 ? wid : rg;
  auto reduce = [&](float (&p)[V], float* buf) {
    for (int o = ncp; o < 64; o <<= 1)
#pragma unroll
      for (int i = 0; i < V; ++i) p[i] += __shfl_xor(p[i], o, 64);
    if (ncp >= 64 || lane < ncp) stV<V>(buf + mypart * ncp * V + c0, p);
    __syncthreads();
#pragma unroll
    for (int i = 0; i < V; ++i) p[i] = 0.f;
    for (int j = 0; j < npart; ++j) {
      float t[V];
      ldV<V>(buf + j * ncp * V + c0, t);
#pragma unroll
      for (int i = 0; i < V; ++i) p[i] += t[i];
    }
  };
  __syncthreads();
  const float g = gb[0], beta = gb[1];
  float p[V];
#pragma unroll
  for (int i = 0; i < V; ++i) p[i] = 0.f;
#pragma unroll
  for (int u = 0; u < RPT; ++u) {
    const int r = rg + RG * u;
    const float kr = r < d ? ks[r] : 0.f;
#pragma unroll
    for (int i = 0; i < V; ++i) {
      S[u][i] *= g;
      p[i] = fmaf(S[u][i], kr, p[i]);
    }
  }
  reduce(p, part[0]);
  float uu[V];
#pragma unroll
  for (int i = 0; i < V; ++i) {
    uu[i] = beta * (vv[i] - p[i]);
    p[i] = 0.f;
  }
#pragma unroll
  for (int u = 0; u < RPT; ++u) {
    const int r = rg + RG * u;
    const float kr = r < d ? ks[r] : 0.f, qr = r < d ? qs[r] : 0.f;
#pragma unroll
    for (int i = 0; i < V; ++i) {
      S[u][i] = fmaf(kr, uu[i], S[u][i]);
      p[i] = fmaf(S[u][i], qr, p[i]);
    }
    if (slot_ok && c_ok && r < d) stV<V>(Sg + (size_t)r * vd + c0, S[u]);
  }
  reduce(p, part[1]);
  float ss = 0.f;
  if (rg == 0 && c_ok) {
#pragma unroll
    for (int i = 0; i < V; ++i) ss = fmaf(p[i], p[i], ss);
  }
  ss = block_sum(ss, red);
  if (rg == 0 && c_ok) {
    const float r = 1.f / sqrtf(ss / (float)vd + eps);
#pragma unroll
    for (int i = 0; i < V; ++i)
      std_(y + (size_t)row * (H * vd) + h * vd + c0 + i,
           p[i] * r * wn[h * vd + c0 + i] * (gt[i] * sigmoid_d(gt[i])));
  }
}

}  // namespace grag

using namespace grag;

#define DT_DISPATCH(dt, ...)                   \
  if ((dt) == 0) {                             \
    using T = bf16;                            \
    __VA_ARGS__                                \
  } else {                                     \
    using T = float;                           \
    __VA_ARGS__                                \
  }

GRAG_API int grag_delta_chunk() { return DC; }
GRAG_API int grag_delta_max_dim() { return DMAX; }
// scratch bytes per chunk and q / k head (per_head 0) or head (1)
GRAG_API int grag_delta_ws_bytes(int d, int dt, int per_head) {
  return per_head ? HB_FLOATS * 4 : 3 * DC * ((d + 31) / 32 * 32) * (dt == 0 ? 2 : 4);
}

// Portions of up to max_q_len tokens: out [T][H * vd] fp32 = the read-outs.  wk / wh: scratch of nchunks rows (of G and H
// blocks of grag_delta_ws_bytes), nchunks >= (all tokens) / DC + nseq.
GRAG_API hipError_t grag_delta_scan(const void* xc, int C, const void* proj, int ld, int boff, int aoff,
                                    const float* a_log, const float* dt_bias, float* state, const int* slots,
                                    const int* q_start, const int* ctx_len, float* out, int nseq, int H, int G, int d,
                                    int vd, int nslots, int dt, void* wk, void* wh, int nchunks, int max_q_len,
                                    hipStream_t st) {
  if (nseq <= 0 || max_q_len <= 0) return hipSuccess;
  const int maxch = (max_q_len + DC - 1) / DC, ntile = (vd + 15) / 16;
  if (d < 1 || vd < 1 || d > DMAX || vd > DMAX || G < 1 || H % G || C < 2 * G * d + H * vd || nseq > 65535 ||
      maxch > 65535 || wk == nullptr || wh == nullptr || ((reinterpret_cast<uintptr_t>(wk) | reinterpret_cast<uintptr_t>(wh)) & 15))
    return hipErrorInvalidValue;
  const int ND = (d + 31) / 32, dp = 32 * ND;
  const int vec = C % 8 == 0 && d % 8 == 0 && (reinterpret_cast<uintptr_t>(xc) & 15) == 0;
  const size_t lk = dp + (dt == 0 ? 8 : 4);
  const size_t kq = 2 * DC * lk * (dt == 0 ? 2 : 4), tri = DC * 68 * sizeof(float);
  const size_t bytes = (kq > tri ? kq : tri) + (2560 + 5 * DC) * sizeof(float);
#define DELTA_SCAN(NDM)                                                                                              \
  hipLaunchKernelGGL((delta_scan_kernel<T, NDM>), grid, dim3(256), 0, st, (const T*)xc, C, state, slots, q_start,    \
                     ctx_len, out, H, G, d, vd, nslots, (const T*)wk, (const float*)wh, nchunks)
  DT_DISPATCH(dt, {
    if (bytes > 48 * 1024) {
      const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(&delta_prep_kernel<T>),
                                               hipFuncAttributeMaxDynamicSharedMemorySize, (int)bytes);
      if (e != hipSuccess) return e;
    }
    hipLaunchKernelGGL(delta_prep_kernel<T>, dim3(H, maxch, nseq), dim3(256), bytes, st, (const T*)xc, C, (const T*)proj,
                       ld, boff, aoff, a_log, dt_bias, q_start, H, G, d, vec, (T*)wk, (float*)wh, nchunks);
    const dim3 grid((unsigned)nseq * H * ntile);
    if (ND <= 2) {
      DELTA_SCAN(2);
    } else if (ND <= 4) {
      DELTA_SCAN(4);
    } else {
      DELTA_SCAN(8);
    }
  })
#undef DELTA_SCAN
  return hipGetLastError();
}

// One token per sequence: y [T][H * vd] in the activation type, the gated RMS norm included.
GRAG_API hipError_t grag_delta_step(const void* xc, int C, const void* proj, int ld, int boff, int aoff, int goff,
                                    const float* a_log, const float* dt_bias, const float* wn, float eps, float* state,
                                    const int* slots, const int* q_start, const int* ctx_len, void* y, int nseq, int H,
                                    int G, int d, int vd, int nslots, int dt, hipStream_t st) {
  if (nseq <= 0) return hipSuccess;
  if (d < 1 || vd < 1 || d > DMAX || vd > DMAX || G < 1 || H % G || C < 2 * G * d + H * vd || nseq > 65535)
    return hipErrorInvalidValue;
  const int V = vd % 4 == 0 && (reinterpret_cast<uintptr_t>(state) & 15) == 0 ? 4 : 1, maxr = V == 4 ? 16 : 64;
  int ncp = 1, nt = 256;
  while (ncp * V < vd) ncp <<= 1;
  while ((d + nt / ncp - 1) / (nt / ncp) > maxr) nt <<= 1;  // (at most 1024: 256 x 256 numbers are 64 a thread)
  const int rpt = (d + nt / ncp - 1) / (nt / ncp);
#define DELTA_STEP(VV, RPT, NT)                                                                                       \
  hipLaunchKernelGGL((delta_step_kernel<T, VV, RPT, NT>), dim3(H, nseq), dim3(nt), 0, st, (const T*)xc, C, (const T*)proj, \
                     ld, boff, aoff, goff, a_log, dt_bias, wn, eps, state, slots, q_start, ctx_len, (T*)y, H, G, d, vd, \
                     nslots, ncp)
  DT_DISPATCH(dt, {
    if (V == 1) {
      if (nt > 256) DELTA_STEP(1, 64, 1024);
      else if (rpt <= 16) DELTA_STEP(1, 16, 256);
      else DELTA_STEP(1, 64, 256);
    } else if (nt > 256) {
      DELTA_STEP(4, 16, 1024);
    } else if (rpt <= 4) {
      DELTA_STEP(4, 4, 256);
    } else if (rpt <= 8) {
      DELTA_STEP(4, 8, 256);
    } else {
      DELTA_STEP(4, 16, 256);
    }
  })
#undef DELTA_STEP
  return hipGetLastError();
}
