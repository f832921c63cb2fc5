// State-space sequence mixer (gfx950): the short causal convolution in front of it and the selective scan.
//   * causal depthwise convolution + SiLU over a column range of a fused projection; the last taps - 1 inputs of every
//     sequence live in a slot-indexed pool, so a prompt may be cut anywhere and decoding continues from it,
//   * the scan: per head a state S [N, P] fp32 with a scalar, input-dependent decay per step,
//       dt_t = softplus(raw_t + bias_h),  S_t = exp(-exp(A_log_h) dt_t) S_(t-1) + dt_t B_t x_t^T,  y_t = S_t^T C_t + D_h x_t
//     (B, C shared by the heads of a group).  Everything between the convolution's output and y is fp32.
//   * the scan with a decay per channel AND state number: per channel c a state of N numbers,
//       dt_t = softplus(W_dt low_t + bias_c),  S_n = exp(dt_t A_(c,n)) S_n + dt_t x_t B_(t,n),  y_t = sum_n S_n C_(t,n) + D_c x_t
//     (low, B, C: one small projection per token, shared by the channels), the output gated by SiLU(z) as it is stored.
// Activations are bf16 or fp32 (dt: 0 = bf16, 1 = fp32).  A sequence whose first token of the step sits at position 0
// starts from zeros instead of its slot's contents, so a slot that is used again needs no reset.
#include "common.h"

GRAG_ERR_UNIT(ssm)

namespace grag {

template <typename T> __device__ __forceinline__ float lds(const T* p);
template <> __device__ __forceinline__ float lds<bf16>(const bf16* p) { return (float)*p; }
template <> __device__ __forceinline__ float lds<float>(const float* p) { return *p; }
template <typename T> __device__ __forceinline__ void sts(T* p, float v);
template <> __device__ __forceinline__ void sts<bf16>(bf16* p, float v) { *p = (bf16)v; }
template <> __device__ __forceinline__ void sts<float>(float* p, float v) { *p = v; }

__device__ __forceinline__ float silu_f(float x) { return x / (1.f + expf(-x)); }
__device__ __forceinline__ float softplus_f(float x) { return x > 20.f ? x : log1pf(expf(x)); }

// softplus out of the hardware's log2 / exp2: log(1 + u), u = e^-|x|, by its series for small u (where 1 + u would round
// u away), else through w = 1 + u with the rounding of w divided out: log(w) u / (w - 1)
__device__ __forceinline__ float softplus_hw(float x) {
  constexpr float LOG2E = 1.4426950408889634f, LN2 = 0.6931471805599453f;
  const float u = __builtin_amdgcn_exp2f(-fabsf(x) * LOG2E);
  const float series = u * fmaf(u, fmaf(u, fmaf(u, fmaf(u, 0.2f, -0.25f), 0.33333334f), -0.5f), 1.f);
  const float w = 1.f + u;
  const float lg = LN2 * __builtin_amdgcn_logf(w) * u * __builtin_amdgcn_rcpf(w - 1.f);
  return fmaxf(x, 0.f) + (u < 0.0625f ? series : lg);
}
// SiLU of a value that is stored as bf16 (hardware exp2 and reciprocal) or as fp32
template <typename T> __device__ __forceinline__ float silu_t(float x) {
  if (sizeof(T) == 2) return x * __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(-1.4426950408889634f * x));
  return silu_f(x);
}

// 4 consecutive elements
template <typename T> __device__ __forceinline__ f32x4_t ld4s(const T* p);
template <> __device__ __forceinline__ f32x4_t ld4s<float>(const float* p) { return *reinterpret_cast<const f32x4_t*>(p); }
template <> __device__ __forceinline__ f32x4_t ld4s<bf16>(const bf16* p) {
  const bf16x4_t v = *reinterpret_cast<const bf16x4_t*>(p);
  return f32x4_t{bits2f(v[0]), bits2f(v[1]), bits2f(v[2]), bits2f(v[3])};
}
template <typename T> __device__ __forceinline__ void st4s(T* p, f32x4_t v);
template <> __device__ __forceinline__ void st4s<float>(float* p, f32x4_t v) { *reinterpret_cast<f32x4_t*>(p) = v; }
template <> __device__ __forceinline__ void st4s<bf16>(bf16* p, f32x4_t v) {
  *reinterpret_cast<bf16x4_t*>(p) = bf16x4_t{f2bits(v[0]), f2bits(v[1]), f2bits(v[2]), f2bits(v[3])};
}

// ------------------------------------------------------------------------------------------------ causal convolution
constexpr int CONV_MAX_TAPS = 16;
constexpr int CONV_TT = 16;  // tokens per workgroup

// out [T][C] = SiLU(b[c] + sum_j w[c][j] in[t - (taps - 1) + j][c]), in = proj columns coff .. coff + C; inputs before
// the portion come from cstate [slots][taps - 1][C] (oldest first), zeros for a sequence that starts at position 0.
// mode bit 0: no SiLU; bit 1: the token's own input is added to the result (in + conv(in)); bit 2 (only when one token
// tile holds every portion, gridDim.y == 1): the thread, which then walks ALL tokens of its (sequence, channel), also
// leaves the last taps - 1 inputs in the pool -- they are the window it ends with -- and no second kernel runs.
// grid (ceil(C / 256), ceil(max_q_len / CONV_TT), nseq).  Without bit 2 the pool is only read here.
template <typename T>
__global__ void __launch_bounds__(256)
causal_conv_kernel(const T* __restrict__ proj, int ld, int coff, int C, int taps, const float* __restrict__ w,
                   const float* __restrict__ b, T* __restrict__ cstate, const int* __restrict__ slots,
                   const int* __restrict__ q_start, const int* __restrict__ ctx_len, T* __restrict__ out, int nslots,
                   int mode) {
  const int seq = blockIdx.z, c = blockIdx.x * 256 + threadIdx.x;
  const int qa = q_start[seq], qlen = q_start[seq + 1] - qa;
  const int t0 = blockIdx.y * CONV_TT;
  if (t0 >= qlen || c >= C) return;
  const bool fresh = ctx_len[seq] - qlen == 0;
  const int slot = slots[seq];
  const bool slot_ok = fresh || index_ok(slot, nslots, ERR_SAMPLER_SLOT);
  const T* st = cstate + (size_t)(slot_ok && !fresh ? slot : 0) * (taps - 1) * C;
  float wt[CONV_MAX_TAPS], win[CONV_MAX_TAPS];
#pragma unroll
  for (int j = 0; j < CONV_MAX_TAPS; ++j) wt[j] = j < taps ? w[(size_t)c * taps + j] : 0.f;
  const float bias = b ? b[c] : 0.f, wlast = w[(size_t)c * taps + taps - 1];
  // win[j] = input at portion index t - (taps - 1) + j; filled for t = t0 (all but the newest), then shifted
#pragma unroll
  for (int j = 0; j < CONV_MAX_TAPS; ++j) {
    win[j] = 0.f;
    if (j < taps - 1) {
      const int s = t0 - (taps - 1) + j;
      if (s >= 0) win[j] = lds(proj + (size_t)(qa + s) * ld + coff + c);
      else if (!fresh && slot_ok) win[j] = lds(st + (size_t)(taps - 1 + s) * C + c);
    }
  }
  const int nt = min(CONV_TT, qlen - t0);
  for (int tt = 0; tt < nt; ++tt) {
    const float cur = lds(proj + (size_t)(qa + t0 + tt) * ld + coff + c);
    float acc = bias;
#pragma unroll
    for (int j = 0; j < CONV_MAX_TAPS; ++j) {
      if (j < taps - 1) acc = fmaf(wt[j], win[j], acc);
    }
    acc = fmaf(wlast, cur, acc);
    if (!(mode & 1)) acc = silu_f(acc);
    if (mode & 2) acc += cur;
    sts(out + (size_t)(qa + t0 + tt) * C + c, acc);
#pragma unroll
    for (int j = 0; j < CONV_MAX_TAPS - 1; ++j) win[j] = j < taps - 2 ? win[j + 1] : j == taps - 2 ? cur : win[j];
  }
  if ((mode & 4) && taps > 1 && index_ok(slot, nslots, ERR_SAMPLER_SLOT)) {
    T* dst = cstate + (size_t)slot * (taps - 1) * C;
#pragma unroll
    for (int j = 0; j < CONV_MAX_TAPS - 1; ++j)
      if (j < taps - 1) sts(dst + (size_t)j * C + c, win[j]);
  }
}

// The same for up to MT taps and rows in groups of four channels (C, ld, coff multiples of 4, aligned pointers): a thread
// owns four channels of a token tile, all of whose inputs are in flight before the first sum.  The weights stand at the
// end of MT places (zeros before them), so every register index is known when the kernel is compiled.
// grid (ceil(C / 1024), ceil(max_q_len / CONV_TT), nseq); the mode bits as above.
template <typename T, int MT>
__global__ void __launch_bounds__(256)
causal_conv_vec_kernel(const T* __restrict__ proj, int ld, int coff, int C, int taps, const float* __restrict__ w,
                       const float* __restrict__ b, T* __restrict__ cstate, const int* __restrict__ slots,
                       const int* __restrict__ q_start, const int* __restrict__ ctx_len, T* __restrict__ out, int nslots,
                       int mode) {
  const int seq = blockIdx.z, c = (blockIdx.x * 256 + threadIdx.x) * 4;
  const int qa = q_start[seq], qlen = q_start[seq + 1] - qa;
  const int t0 = blockIdx.y * CONV_TT;
  if (t0 >= qlen || c >= C) return;
  const bool fresh = ctx_len[seq] - qlen == 0;
  const int slot = slots[seq];
  const bool slot_ok = fresh || index_ok(slot, nslots, ERR_SAMPLER_SLOT);
  const T* st = cstate + (size_t)(slot_ok && !fresh ? slot : 0) * (taps - 1) * C + c;
  const T* in = proj + (size_t)qa * ld + coff + c;
  const int nt = min(CONV_TT, qlen - t0), lead = MT - taps;
  f32x4_t cur[CONV_TT], win[MT - 1];  // the tile's inputs; the MT - 1 inputs before the one at hand, oldest first
#pragma unroll
  for (int tt = 0; tt < CONV_TT; ++tt)
    cur[tt] = tt < nt ? ld4s(in + (size_t)(t0 + tt) * ld) : f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int j = 0; j < MT - 1; ++j) {
    win[j] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    const int s = t0 - (MT - 1) + j;  // token index in the portion
    if (j >= lead) {
      if (s >= 0) win[j] = ld4s(in + (size_t)s * ld);
      else if (!fresh && slot_ok) win[j] = ld4s(st + (size_t)(taps - 1 + s) * C);
    }
  }
  float wt[MT][4];
#pragma unroll
  for (int j = 0; j < MT; ++j)
#pragma unroll
    for (int v = 0; v < 4; ++v) wt[j][v] = j >= lead ? w[(size_t)(c + v) * taps + j - lead] : 0.f;
  const f32x4_t bias = b ? *reinterpret_cast<const f32x4_t*>(b + c) : f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int tt = 0; tt < CONV_TT; ++tt) {
    if (tt < nt) {
      f32x4_t acc = bias;
#pragma unroll
      for (int j = 0; j < MT - 1; ++j)
#pragma unroll
        for (int v = 0; v < 4; ++v) acc[v] = fmaf(wt[j][v], win[j][v], acc[v]);
#pragma unroll
      for (int v = 0; v < 4; ++v) acc[v] = fmaf(wt[MT - 1][v], cur[tt][v], acc[v]);
      if (!(mode & 1)) {
#pragma unroll
        for (int v = 0; v < 4; ++v) acc[v] = silu_t<T>(acc[v]);
      }
      if (mode & 2) acc += cur[tt];
      st4s(out + (size_t)(qa + t0 + tt) * C + c, acc);
#pragma unroll
      for (int j = 0; j < MT - 2; ++j) win[j] = win[j + 1];
      win[MT - 2] = cur[tt];
    }
  }
  if ((mode & 4) && taps > 1 && index_ok(slot, nslots, ERR_SAMPLER_SLOT)) {  // (t0 is 0: one tile holds the portion)
    T* dst = cstate + (size_t)slot * (taps - 1) * C + c;
#pragma unroll
    for (int j = 0; j < MT - 1; ++j) {
      if (j < lead) continue;
      st4s(dst + (size_t)(j - lead) * C, win[j]);
    }
  }
}

// the pool after the step: the last taps - 1 inputs of every sequence (runs after the kernel above, on the same stream).
// grid (ceil(C / 256), nseq): a thread reads all it needs of its channel before it writes.
template <typename T>
__global__ void __launch_bounds__(256)
conv_state_kernel(const T* __restrict__ proj, int ld, int coff, int C, int taps, T* __restrict__ cstate,
                  const int* __restrict__ slots, const int* __restrict__ q_start, const int* __restrict__ ctx_len,
                  int nslots) {
  const int seq = blockIdx.y, c = blockIdx.x * 256 + threadIdx.x;
  const int qa = q_start[seq], qlen = q_start[seq + 1] - qa;
  if (qlen <= 0 || c >= C || taps < 2) return;
  const bool fresh = ctx_len[seq] - qlen == 0;
  const int slot = slots[seq];
  if (!index_ok(slot, nslots, ERR_SAMPLER_SLOT)) return;
  T* st = cstate + (size_t)slot * (taps - 1) * C;
  float v[CONV_MAX_TAPS];
#pragma unroll
  for (int j = 0; j < CONV_MAX_TAPS; ++j) {
    v[j] = 0.f;
    if (j < taps - 1) {
      const int s = qlen - (taps - 1) + j;
      if (s >= 0) v[j] = lds(proj + (size_t)(qa + s) * ld + coff + c);
      else if (!fresh) v[j] = lds(st + (size_t)(taps - 1 + s) * C + c);
    }
  }
#pragma unroll
  for (int j = 0; j < CONV_MAX_TAPS; ++j)
    if (j < taps - 1) sts(st + (size_t)j * C + c, v[j]);
}

// ------------------------------------------------------------------------------------------------ selective scan
// xbc [T][C]: x heads at column 0 (H x P), B groups at boff (G x N), C groups at coff (G x N) -- the convolution's
// output.  dt raw at column dtoff + h of proj [T][ld].  state [slots][H][N][P] fp32, out [T][H * P] fp32.
// grid (H, nseq); thread j < P owns column j of S in registers (NMAX rows).  Tokens are walked in order, TB at a time
// through LDS.  Long portions are cut into chunks of SSM_CHUNK tokens that run side by side, as the decay scan does:
//   MODE 0  the whole portion in one workgroup, from and to the slot's state;
//   MODE 1  grid.z = chunk: the chunk's own contribution from a zero state -> ws [nseq * maxchunks][H][N][P], and the
//           product of the chunk's decays -> wa [nseq * maxchunks][H];
//   (ssm_chunk_prefix_kernel turns ws[c] into the state at the START of chunk c and stores the final state;)
//   MODE 2  grid.z = chunk: the outputs of the chunk's tokens, from the chunk-start state in ws.
constexpr int SSM_CHUNK = 64;

template <typename T, int NMAX, int MODE>
__global__ void __launch_bounds__(256)
ssm_scan_kernel(const T* __restrict__ xbc, int C, int boff, int coff, const T* __restrict__ proj, int ld, int dtoff,
                const float* __restrict__ dt_bias, const float* __restrict__ A_log, const float* __restrict__ Dv,
                float* __restrict__ state, const int* __restrict__ slots, const int* __restrict__ q_start,
                const int* __restrict__ ctx_len, float* __restrict__ out, int H, int G, int N, int P, int nslots,
                float* __restrict__ ws, float* __restrict__ wa, int maxchunks) {
  constexpr int TB = 16;
  extern __shared__ __attribute__((aligned(16))) float smem[];  // [TB][2][np] B*dt | C, [TB][P] x, [TB] decay
  const int np = (N + 3) & ~3;
  float* xs = smem + TB * 2 * np;
  float* as = xs + TB * P;
  const int seq = blockIdx.y, h = blockIdx.x, g = h / (H / G);
  int qa = q_start[seq], qlen = q_start[seq + 1] - qa;
  if (qlen <= 0) return;
  const int j = threadIdx.x;
  const bool fresh = ctx_len[seq] - qlen == 0;
  const int slot = MODE == 0 ? slots[seq] : 0;
  const bool slot_ok = MODE == 0 ? index_ok(slot, nslots, ERR_SAMPLER_SLOT) : true;
  float* Sg = state + (((size_t)(slot_ok ? slot : 0) * H + h) * N) * P;
  int chunk = 0;
  if (MODE != 0) {
    chunk = blockIdx.z;
    if (chunk * SSM_CHUNK >= qlen) return;
    qa += chunk * SSM_CHUNK;
    qlen = min(SSM_CHUNK, qlen - chunk * SSM_CHUNK);
    Sg = ws + (((size_t)(seq * maxchunks + chunk) * H + h) * N) * P;
  }
  const float rate = expf(A_log[h]), bias = dt_bias[h], dsk = Dv[h];
  float S[NMAX];
#pragma unroll
  for (int i = 0; i < NMAX; ++i) {
    if (MODE == 0) S[i] = (!fresh && slot_ok && i < N && j < P) ? Sg[(size_t)i * P + j] : 0.f;
    if (MODE == 1) S[i] = 0.f;
    if (MODE == 2) S[i] = (i < N && j < P) ? Sg[(size_t)i * P + j] : 0.f;
  }
  float aprod = 1.f;
  for (int t0 = 0; t0 < qlen; t0 += TB) {
    const int nb = min(TB, qlen - t0);
    __syncthreads();
    if (threadIdx.x < nb) {
      const float dtv = softplus_f(lds(proj + (size_t)(qa + t0 + threadIdx.x) * ld + dtoff + h) + bias);
      as[threadIdx.x] = expf(-rate * dtv);
      as[TB + threadIdx.x] = dtv;
    }
    __syncthreads();
    for (int idx = threadIdx.x; idx < nb * 2 * N; idx += blockDim.x) {
      const int tt = idx / (2 * N), r = idx - tt * 2 * N;
      const int which = r / N, i = r - which * N;  // 0: B (scaled by dt), 1: C
      const float val = lds(xbc + (size_t)(qa + t0 + tt) * C + (which ? coff : boff) + g * N + i);
      smem[(tt * 2 + which) * np + i] = which ? val : val * as[TB + tt];
    }
    for (int idx = threadIdx.x; idx < nb * P; idx += blockDim.x) {
      const int tt = idx / P, i = idx - tt * P;
      xs[idx] = lds(xbc + (size_t)(qa + t0 + tt) * C + h * P + i);
    }
    __syncthreads();
    if (j < P) {
      for (int tt = 0; tt < nb; ++tt) {
        const float xj = xs[tt * P + j], a = as[tt];
        const f32x4_t* bs = reinterpret_cast<const f32x4_t*>(smem + tt * 2 * np);
        const f32x4_t* cs = reinterpret_cast<const f32x4_t*>(smem + (tt * 2 + 1) * np);
        float y = 0.f;
#pragma unroll
        for (int i4 = 0; i4 < NMAX / 4; ++i4) {
          if (i4 * 4 < N) {
            const f32x4_t b4 = bs[i4];
            const f32x4_t c4 = MODE != 1 ? cs[i4] : f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int e = 0; e < 4; ++e) {
              const int i = i4 * 4 + e;
              if (i < N) {
                S[i] = fmaf(a, S[i], b4[e] * xj);
                if (MODE != 1) y = fmaf(S[i], c4[e], y);
              }
            }
          }
        }
        if (MODE == 1) aprod *= a;
        if (MODE != 1) out[(size_t)(qa + t0 + tt) * (size_t)(H * P) + h * P + j] = fmaf(dsk, xj, y);
      }
    }
  }
  if (MODE != 2 && slot_ok && j < P) {
#pragma unroll
    for (int i = 0; i < NMAX; ++i)
      if (i < N) Sg[(size_t)i * P + j] = S[i];
  }
  if (MODE == 1 && j == 0) wa[(size_t)(seq * maxchunks + chunk) * H + h] = aprod;
}

// ws[seq, c] (chunk c's own contribution) -> the state at the start of chunk c; the slot's state <- the state after the
// last chunk.  grid (H, nseq, ceil(N * P / 256)): one thread per state element.
__global__ void ssm_chunk_prefix_kernel(float* __restrict__ state, const int* __restrict__ slots,
                                        const int* __restrict__ q_start, const int* __restrict__ ctx_len,
                                        float* __restrict__ ws, const float* __restrict__ wa, int maxchunks, int H,
                                        int NP, int nslots) {
  const int seq = blockIdx.y, h = blockIdx.x;
  const int qlen = q_start[seq + 1] - q_start[seq];
  if (qlen <= 0) return;
  const bool fresh = ctx_len[seq] - qlen == 0;
  const int slot = slots[seq];
  if (!index_ok(slot, nslots, ERR_SAMPLER_SLOT)) return;
  const int e = blockIdx.z * blockDim.x + threadIdx.x;
  if (e >= NP) return;
  float* Sg = state + ((size_t)slot * H + h) * NP;
  const int nch = (qlen + SSM_CHUNK - 1) / SSM_CHUNK;
  const size_t cs = (size_t)H * NP;
  float S = fresh ? 0.f : Sg[e];
  float* w = ws + ((size_t)seq * maxchunks * H + h) * NP + e;
  const float* a = wa + (size_t)seq * maxchunks * H + h;
  for (int c = 0; c < nch; ++c) {
    const float u = w[c * cs];
    w[c * cs] = S;
    S = fmaf(a[(size_t)c * H], S, u);
  }
  Sg[e] = S;
}

// ------------------------------------------------------------------------------------------------ per-channel scan
// xc [T][inner]: the convolution's output; low [T][low_ld]: step-size numbers (R) | B (N) | C (N); wdt [inner][Rp], the step
// sizes' matrix, its rows padded with zeros to Rp (a multiple of 32); A [inner][N] fp32 (negative); z = columns zoff ..
// of proj [T][ld].  state [slots][inner][N] fp32; out [T][inner] = y * SiLU(z).  grid (ceil(inner / 64), nseq, chunks),
// 256 threads: thread (channel tid / 4, lane part tid % 4) keeps the state numbers 4 (part + 4 j) .. + 3, j < NPT / 4, in
// registers (4 NPT >= N; numbers past N have B = C = 0).  Tokens are walked SC_TB at a time:
//   staging   wave w forms the step sizes of its 16 channels for the 16 tokens -- for bf16 one 16 x 16 matrix-core tile
//             (operand lane: row lane % 16, k = 8 (lane / 16) .. + 7; result lane: tokens 4 (lane / 16) + i, channel
//             lane % 16) -- and leaves (dt log2 e, dt x) per (token, channel) in LDS, beside the tokens' B and C rows;
//   walk      every thread updates its numbers; the four parts of a channel add up their share of y;
//   store     the lane that formed dt adds D x, gates and stores.
// Long portions are cut into chunks of `chunk` tokens (a multiple of SC_TB) that run side by side:
//   MODE 0  the whole portion, from and to the slot's state;
//   MODE 1  grid.z = chunk: the chunk's own contribution from a zero state -> ws [nseq * maxchunks][inner][N], and the sum
//           of its step sizes (times log2 e) -> wa [nseq * maxchunks][inner];
//   (chan_chunk_prefix_kernel turns ws[c] into the state at the START of chunk c and stores the final state;)
//   MODE 2  grid.z = chunk: the outputs of the chunk's tokens, from the chunk-start state in ws.
constexpr int SC_TB = 16, SC_CH = 64;

// sum over the 4 lanes of a channel, in every lane
__device__ __forceinline__ float quad_sum(float v) {
  v += __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), 0xB1, 0xf, 0xf, true));  // lanes 1 0 3 2
  v += __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), 0x4E, 0xf, 0xf, true));  // lanes 2 3 0 1
  return v;
}

template <typename T, int NPT, int MODE>
__global__ void __launch_bounds__(256)
chan_scan_kernel(const T* __restrict__ xc, const T* __restrict__ low, int low_ld, const T* __restrict__ wdt, int R, int Rp,
                 const float* __restrict__ dt_bias, const float* __restrict__ A, const float* __restrict__ Dv,
                 const T* __restrict__ proj, int ld, int zoff, float* __restrict__ state, const int* __restrict__ slots,
                 const int* __restrict__ q_start, const int* __restrict__ ctx_len, T* __restrict__ out, int inner, int N,
                 int nslots, float* __restrict__ ws, float* __restrict__ wa, int chunk_len, int maxchunks) {
  constexpr float LOG2E = 1.4426950408889634f;
  constexpr int NP = 4 * NPT;
  typedef float f32x2_t __attribute__((ext_vector_type(2)));
  __shared__ __attribute__((aligned(16))) float bc[SC_TB][2][NP];
  __shared__ __attribute__((aligned(16))) f32x2_t sd[SC_TB][SC_CH];
  __shared__ float sy[MODE == 1 ? 1 : SC_TB][SC_CH];
  const int seq = blockIdx.y, c0 = blockIdx.x * SC_CH;
  int qa = q_start[seq], qlen = q_start[seq + 1] - qa;
  if (qlen <= 0) return;
  const bool fresh = ctx_len[seq] - qlen == 0;
  const int slot = MODE == 0 ? slots[seq] : 0;
  const bool slot_ok = MODE == 0 ? index_ok(slot, nslots, ERR_SAMPLER_SLOT) : true;
  float* Sb = state + (size_t)(slot_ok ? slot : 0) * inner * N;
  int chunk = 0;
  if (MODE != 0) {
    chunk = blockIdx.z;
    if (chunk * chunk_len >= qlen) return;
    qa += chunk * chunk_len;
    qlen = min(chunk_len, qlen - chunk * chunk_len);
    Sb = ws + (size_t)(seq * maxchunks + chunk) * inner * N;
  }
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6, ql = lane & 15, quad = lane >> 4;
  // walk role: channel ch, part of its numbers
  const int cl = threadIdx.x >> 2, part = threadIdx.x & 3, ch = c0 + cl;
  const bool ch_ok = ch < inner;
  float S[NPT], a2[NPT];
  const bool vecn = (N & 3) == 0;
#pragma unroll
  for (int j = 0; j < NPT / 4; ++j) {
    const int n0 = 4 * (part + 4 * j);
    f32x4_t av = f32x4_t{0.f, 0.f, 0.f, 0.f}, sv = av;
    if (ch_ok && n0 < N) {
      const float* ap = A + (size_t)ch * N + n0;
      const float* sp = Sb + (size_t)ch * N + n0;
      const bool use = MODE == 2 || (MODE == 0 && !fresh && slot_ok);
      if (vecn) {
        av = *reinterpret_cast<const f32x4_t*>(ap);
        if (use) sv = *reinterpret_cast<const f32x4_t*>(sp);
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (n0 + e < N) {
            av[e] = ap[e];
            if (use) sv[e] = sp[e];
          }
      }
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      a2[4 * j + e] = av[e];
      S[4 * j + e] = sv[e];
    }
  }
  // staging role: channel sc of tokens 4 quad + i
  const int sc = c0 + 16 * wid + ql;
  const bool sc_ok = sc < inner;
  const int scc = sc_ok ? sc : 0;  // (loads of lanes past the last channel or token go to a valid place and are not used)
  const float bias = sc_ok ? dt_bias[sc] : 0.f, dsk = sc_ok ? Dv[sc] : 0.f;
  const T* wrow = wdt + (size_t)scc * Rp;
  constexpr int NW = 8;  // matrix fragments kept in registers (R up to 256); the rest is read again per tile
  constexpr int NB = NPT <= 8 ? SC_TB * 2 * NP / 256 : 1;  // B / C elements per thread fetched ahead
  bf16x8_t wf[NW], lf[NW];
  T xn[4], zn[4], bn[NB];  // (as they are read: nothing waits for them before the walk is over)
  if (sizeof(T) == 2) {
#pragma unroll
    for (int k = 0; k < NW; ++k)
      wf[k] = 32 * k < Rp ? *reinterpret_cast<const bf16x8_t*>(wrow + 32 * k + 8 * quad) : bf16x8_t{0, 0, 0, 0, 0, 0, 0, 0};
  }
  // rows of low are padded to a multiple of 8, so a vector that starts below R lies in its row; one that starts past R
  // meets zeros of the matrix and is taken from the row's start instead
  auto lfrag = [&](const T* lrow, int k) {
    return *reinterpret_cast<const bf16x8_t*>(lrow + (32 * k + 8 * quad < R ? 32 * k + 8 * quad : 0));
  };
  auto bc_at = [&](int t0, int nb, int idx) {
    const int t = idx / (2 * NP), r = idx - t * 2 * NP, n = r & (NP - 1);
    const bool ok = t < nb && n < N;
    return low[(size_t)(qa + t0 + (ok ? t : 0)) * low_ld + R + (r < NP ? 0 : N) + (ok ? n : 0)];
  };
  auto bc_put = [&](int nb, int idx, T v) {  // (past the last token or state number: zeros)
    (&bc[0][0][0])[idx] = idx / (2 * NP) < nb && (idx & (NP - 1)) < N ? (float)v : 0.f;
  };
  auto fetch = [&](int t0) {  // a tile's global reads
    const int nb = min(SC_TB, qlen - t0);
    if (sizeof(T) == 2) {
      const T* lrow = low + (size_t)(qa + t0 + min(ql, nb - 1)) * low_ld;
#pragma unroll
      for (int k = 0; k < NW; ++k)
        if (32 * k < Rp) lf[k] = lfrag(lrow, k);
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const size_t row = qa + t0 + min(4 * quad + i, nb - 1);
      xn[i] = xc[row * inner + scc];
      if (MODE != 1) zn[i] = proj[row * ld + zoff + scc];
    }
    if (NPT <= 8) {
#pragma unroll
      for (int u = 0; u < NB; ++u) bn[u] = bc_at(t0, nb, threadIdx.x + 256 * u);
    }
  };
  fetch(0);
  float dtsum = 0.f;
  for (int t0 = 0; t0 < qlen; t0 += SC_TB) {
    const int nb = min(SC_TB, qlen - t0);
    // step sizes before softplus
    float dv[4] = {bias, bias, bias, bias};
    if (sizeof(T) == 2) {
      f32x4_t acc = f32x4_t{bias, bias, bias, bias};
#pragma unroll
      for (int k = 0; k < NW; ++k)
        if (32 * k < Rp) acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(lf[k], wf[k], acc, 0, 0, 0);
      const T* lrow = low + (size_t)(qa + t0 + min(ql, nb - 1)) * low_ld;
      for (int k = NW; 32 * k < Rp; ++k)
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
            lfrag(lrow, k), *reinterpret_cast<const bf16x8_t*>(wrow + 32 * k + 8 * quad), acc, 0, 0, 0);
#pragma unroll
      for (int i = 0; i < 4; ++i) dv[i] = acc[i];
    } else {
      for (int k = 0; k < R; ++k) {
        const float w = lds(wrow + k);
#pragma unroll
        for (int i = 0; i < 4; ++i)
          dv[i] = fmaf(lds(low + (size_t)(qa + t0 + min(4 * quad + i, nb - 1)) * low_ld + k), w, dv[i]);
      }
    }
    float xv[4], zv[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      xv[i] = (float)xn[i];
      if (MODE != 1) zv[i] = (float)zn[i];
    }
    __syncthreads();  // the tile before is consumed
    // (a token past the portion's end leaves the state as it is: dt = 0, B = C = 0)
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const float dt = 4 * quad + i < nb ? softplus_hw(dv[i]) : 0.f;
      sd[4 * quad + i][16 * wid + ql] = f32x2_t{dt * LOG2E, dt * xv[i]};
    }
    if (NPT <= 8) {
#pragma unroll
      for (int u = 0; u < NB; ++u) bc_put(nb, threadIdx.x + 256 * u, bn[u]);
    } else {
      for (int idx = threadIdx.x; idx < SC_TB * 2 * NP; idx += 256) bc_put(nb, idx, bc_at(t0, nb, idx));
    }
    __syncthreads();
    if (t0 + SC_TB < qlen) fetch(t0 + SC_TB);  // in flight during the walk
    for (int t4 = 0; t4 < nb; t4 += 4) {
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const int t = t4 + u;
        const f32x2_t d = sd[t][cl];
        float y = 0.f;
#pragma unroll
        for (int j = 0; j < NPT / 4; ++j) {
          const f32x4_t b4 = *reinterpret_cast<const f32x4_t*>(&bc[t][0][4 * (part + 4 * j)]);
#pragma unroll
          for (int e = 0; e < 4; ++e)
            S[4 * j + e] = fmaf(__builtin_amdgcn_exp2f(d[0] * a2[4 * j + e]), S[4 * j + e], d[1] * b4[e]);
          if (MODE != 1) {
            const f32x4_t c4 = *reinterpret_cast<const f32x4_t*>(&bc[t][1][4 * (part + 4 * j)]);
#pragma unroll
            for (int e = 0; e < 4; ++e) y = fmaf(S[4 * j + e], c4[e], y);
          }
        }
        if (MODE == 1) dtsum += d[0];
        else sy[t][cl] = quad_sum(y);
      }
    }
    if (MODE != 1) {
      __syncthreads();
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int t = 4 * quad + i;
        const float o = fmaf(dsk, xv[i], sy[t][16 * wid + ql]) * silu_t<T>(zv[i]);
        if (t < nb && sc_ok) sts(out + (size_t)(qa + t0 + t) * inner + sc, o);
      }
    }
  }
  if (MODE != 2 && slot_ok && ch_ok) {
#pragma unroll
    for (int j = 0; j < NPT / 4; ++j) {
      const int n0 = 4 * (part + 4 * j);
      if (n0 >= N) continue;
      float* sp = Sb + (size_t)ch * N + n0;
      if (vecn) {
        *reinterpret_cast<f32x4_t*>(sp) = f32x4_t{S[4 * j], S[4 * j + 1], S[4 * j + 2], S[4 * j + 3]};
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (n0 + e < N) sp[e] = S[4 * j + e];
      }
    }
  }
  if (MODE == 1 && part == 0 && ch_ok) wa[(size_t)(seq * maxchunks + chunk) * inner + ch] = dtsum;
}

// One token per sequence (decode rows): the same with sequences in the place of tokens.  grid (ceil(inner / 64),
// ceil(nseq / SB)): a workgroup takes 64 channels of SB <= SC_TB sequences, so the step-size matrix is read once for all of
// them.  States travel G sequences at a time, the next group's loads in flight during the sums of the one before.
template <typename T, int NPT, int G>
__global__ void __launch_bounds__(256)
chan_step_kernel(const T* __restrict__ xc, const T* __restrict__ low, int low_ld, const T* __restrict__ wdt, int R, int Rp,
                 const float* __restrict__ dt_bias, const float* __restrict__ A, const float* __restrict__ Dv,
                 const T* __restrict__ proj, int ld, int zoff, float* __restrict__ state, const int* __restrict__ slots,
                 const int* __restrict__ q_start, const int* __restrict__ ctx_len, T* __restrict__ out, int nseq, int SB,
                 int inner, int N, int nslots) {
  constexpr float LOG2E = 1.4426950408889634f;
  constexpr int NP = 4 * NPT;
  typedef float f32x2_t __attribute__((ext_vector_type(2)));
  __shared__ __attribute__((aligned(16))) float bc[SC_TB][2][NP];
  __shared__ __attribute__((aligned(16))) f32x2_t sd[SC_TB][SC_CH];
  __shared__ float sy[SC_TB][SC_CH];
  __shared__ int srow[SC_TB], sslot[SC_TB], sfresh[SC_TB];  // token row (-1: no token), slot (-1: none), starts from zeros
  const int s0 = blockIdx.y * SB, ns = min(SB, nseq - s0), c0 = blockIdx.x * SC_CH;
  if (threadIdx.x < SC_TB) {
    int row = -1, slot = -1, fresh = 1;
    if (threadIdx.x < ns) {
      const int s = s0 + threadIdx.x, qa = q_start[s];
      if (q_start[s + 1] > qa) {
        row = qa;
        fresh = ctx_len[s] == 1;
        slot = slots[s];
        if (!index_ok(slot, nslots, ERR_SAMPLER_SLOT)) slot = -1;
      }
    }
    srow[threadIdx.x] = row;
    sslot[threadIdx.x] = slot;
    sfresh[threadIdx.x] = fresh;
  }
  const int lane = threadIdx.x & 63, wid = threadIdx.x >> 6, ql = lane & 15, quad = lane >> 4;
  const int cl = threadIdx.x >> 2, part = threadIdx.x & 3, ch = c0 + cl;
  const bool ch_ok = ch < inner, vecn = (N & 3) == 0;
  float a2[NPT];
#pragma unroll
  for (int j = 0; j < NPT; ++j) {
    const int n = 4 * (part + 4 * (j >> 2)) + (j & 3);
    a2[j] = ch_ok && n < N ? A[(size_t)ch * N + n] : 0.f;
  }
  __syncthreads();
  auto load = [&](int i, float (&S)[NPT]) {
    const bool use = i < ns && ch_ok && sslot[i < SC_TB ? i : 0] >= 0 && !sfresh[i < SC_TB ? i : 0];
    const float* sp = state + ((size_t)(use ? sslot[i] : 0) * inner + (use ? ch : 0)) * N;
#pragma unroll
    for (int j = 0; j < NPT / 4; ++j) {
      const int n0 = 4 * (part + 4 * j);
      f32x4_t v = f32x4_t{0.f, 0.f, 0.f, 0.f};
      if (use && n0 < N) {
        if (vecn) {
          v = *reinterpret_cast<const f32x4_t*>(sp + n0);
        } else {
#pragma unroll
          for (int e = 0; e < 4; ++e)
            if (n0 + e < N) v[e] = sp[n0 + e];
        }
      }
#pragma unroll
      for (int e = 0; e < 4; ++e) S[4 * j + e] = v[e];
    }
  };
  float S[G][NPT], Sn[G][NPT];
#pragma unroll
  for (int g = 0; g < G; ++g) load(g, S[g]);
  // step sizes of the wave's 16 channels for all the sequences
  const int sc = c0 + 16 * wid + ql;
  const bool sc_ok = sc < inner;
  const float bias = sc_ok ? dt_bias[sc] : 0.f, dsk = sc_ok ? Dv[sc] : 0.f;
  const T* wrow = wdt + (size_t)(sc_ok ? sc : 0) * Rp;
  float dv[4] = {bias, bias, bias, bias};
  if (sizeof(T) == 2) {
    f32x4_t acc = f32x4_t{bias, bias, bias, bias};
    const T* lrow = low + (size_t)max(srow[ql], 0) * low_ld;
    for (int k0 = 0; 32 * k0 < Rp; k0 += 4) {  // four fragments of both operands in flight (past R: zeros of the matrix)
      bf16x8_t fa[4], fb[4];
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        const int o = 32 * (k0 + u) + 8 * quad;
        fa[u] = *reinterpret_cast<const bf16x8_t*>(lrow + (o < R ? o : 0));
        fb[u] = o < Rp ? *reinterpret_cast<const bf16x8_t*>(wrow + o) : bf16x8_t{0, 0, 0, 0, 0, 0, 0, 0};
      }
#pragma unroll
      for (int u = 0; u < 4; ++u) acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fa[u], fb[u], acc, 0, 0, 0);
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) dv[i] = acc[i];
  } else {
    for (int k = 0; k < R; ++k) {
      const float w = lds(wrow + k);
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int r = srow[4 * quad + i];
        dv[i] = fmaf(lds(low + (size_t)(r < 0 ? 0 : r) * low_ld + k), w, dv[i]);
      }
    }
  }
  float xv[4];
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int r = srow[4 * quad + i];
    xv[i] = r >= 0 && sc_ok ? lds(xc + (size_t)r * inner + sc) : 0.f;
    const float dt = softplus_hw(dv[i]);
    sd[4 * quad + i][16 * wid + ql] = f32x2_t{dt * LOG2E, dt * xv[i]};
  }
  for (int idx = threadIdx.x; idx < ns * 2 * NP; idx += 256) {
    const int i = idx / (2 * NP), r = idx - i * 2 * NP, n = r & (NP - 1), row = srow[i];
    bc[i][r / NP][n] = row >= 0 && n < N ? lds(low + (size_t)row * low_ld + R + (r < NP ? 0 : N) + n) : 0.f;
  }
  __syncthreads();
  for (int i0 = 0; i0 < ns; i0 += G) {
    if (i0 + G < ns) {
#pragma unroll
      for (int g = 0; g < G; ++g) load(i0 + G + g, Sn[g]);
    }
#pragma unroll
    for (int g = 0; g < G; ++g) {
      const int i = i0 + g;
      if (i >= ns) break;
      const f32x2_t d = sd[i][cl];
      float y = 0.f;
#pragma unroll
      for (int j = 0; j < NPT / 4; ++j) {
        const f32x4_t b4 = *reinterpret_cast<const f32x4_t*>(&bc[i][0][4 * (part + 4 * j)]);
        const f32x4_t c4 = *reinterpret_cast<const f32x4_t*>(&bc[i][1][4 * (part + 4 * j)]);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          S[g][4 * j + e] = fmaf(__builtin_amdgcn_exp2f(d[0] * a2[4 * j + e]), S[g][4 * j + e], d[1] * b4[e]);
          y = fmaf(S[g][4 * j + e], c4[e], y);
        }
      }
      sy[i][cl] = quad_sum(y);
      if (ch_ok && sslot[i] >= 0) {
        float* sp = state + ((size_t)sslot[i] * inner + ch) * N;
#pragma unroll
        for (int j = 0; j < NPT / 4; ++j) {
          const int n0 = 4 * (part + 4 * j);
          if (n0 >= N) continue;
          if (vecn) {
            *reinterpret_cast<f32x4_t*>(sp + n0) = f32x4_t{S[g][4 * j], S[g][4 * j + 1], S[g][4 * j + 2], S[g][4 * j + 3]};
          } else {
#pragma unroll
            for (int e = 0; e < 4; ++e)
              if (n0 + e < N) sp[n0 + e] = S[g][4 * j + e];
          }
        }
      }
    }
#pragma unroll
    for (int g = 0; g < G; ++g)
#pragma unroll
      for (int j = 0; j < NPT; ++j) S[g][j] = Sn[g][j];
  }
  __syncthreads();
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int r = srow[4 * quad + i];
    if (r >= 0 && sc_ok) {
      const float zv = lds(proj + (size_t)r * ld + zoff + sc);
      sts(out + (size_t)r * inner + sc, fmaf(dsk, xv[i], sy[4 * quad + i][16 * wid + ql]) * silu_t<T>(zv));
    }
  }
}

// ws[seq, c] (chunk c's own contribution) -> the state at the start of chunk c; the slot's state <- the state after the
// last chunk.  grid (ceil(inner * N / 256), nseq): one thread per state number.
__global__ void chan_chunk_prefix_kernel(float* __restrict__ state, const int* __restrict__ slots,
                                         const int* __restrict__ q_start, const int* __restrict__ ctx_len,
                                         const float* __restrict__ A, float* __restrict__ ws, const float* __restrict__ wa,
                                         int chunk_len, int maxchunks, int inner, int N, int nslots) {
  const int seq = blockIdx.y, e = blockIdx.x * 256 + threadIdx.x;
  const int qlen = q_start[seq + 1] - q_start[seq];
  if (qlen <= 0 || e >= inner * N) return;
  const bool fresh = ctx_len[seq] - qlen == 0;
  const int slot = slots[seq];
  if (!index_ok(slot, nslots, ERR_SAMPLER_SLOT)) return;
  float* Sg = state + (size_t)slot * inner * N + e;
  const int nch = (qlen + chunk_len - 1) / chunk_len, c = e / N;
  const float a = A[e];
  float S = fresh ? 0.f : *Sg;
  float* w = ws + (size_t)seq * maxchunks * inner * N + e;
  const float* d = wa + (size_t)seq * maxchunks * inner + c;
  for (int k = 0; k < nch; ++k) {
    const float u = w[(size_t)k * inner * N];
    w[(size_t)k * inner * N] = S;
    S = fmaf(__builtin_amdgcn_exp2f(d[(size_t)k * inner] * a), S, u);
  }
  *Sg = S;
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

GRAG_API int grag_conv_max_taps() { return CONV_MAX_TAPS; }

// update != 0: the pool is brought up to date after the convolution (one call per step and layer run)
GRAG_API hipError_t grag_causal_conv(const void* proj, int ld, int coff, int C, int taps, const float* w, const float* b,
                                     void* cstate, const int* slots, const int* q_start, const int* ctx_len, void* out,
                                     int nseq, int max_q_len, int nslots, int dt, int mode, hipStream_t st) {
  if (nseq <= 0 || max_q_len <= 0) return hipSuccess;
  if (taps < 1 || taps > CONV_MAX_TAPS || C <= 0 || nseq > 65535) return hipErrorInvalidValue;
  const dim3 grid((C + 255) / 256, (max_q_len + CONV_TT - 1) / CONV_TT, nseq);
  if (grid.y > 65535) return hipErrorInvalidValue;
  const bool one_tile = grid.y == 1;  // every portion in one token tile: the convolution's threads update the pool
  mode = (mode & 3) | (one_tile ? 4 : 0);
  const uintptr_t amask = dt == 0 ? 7 : 15;
  const bool vec = C % 4 == 0 && ld % 4 == 0 && coff % 4 == 0 && taps <= 4 && (reinterpret_cast<uintptr_t>(b) & 15) == 0 &&
                   ((reinterpret_cast<uintptr_t>(proj) | reinterpret_cast<uintptr_t>(cstate) |
                     reinterpret_cast<uintptr_t>(out)) & amask) == 0;
  DT_DISPATCH(dt, {
    if (vec)
      hipLaunchKernelGGL((causal_conv_vec_kernel<T, 4>), dim3((C / 4 + 255) / 256, grid.y, nseq), dim3(256), 0, st,
                         (const T*)proj, ld, coff, C, taps, w, b, (T*)cstate, slots, q_start, ctx_len, (T*)out, nslots, mode);
    else
      hipLaunchKernelGGL(causal_conv_kernel<T>, grid, dim3(256), 0, st, (const T*)proj, ld, coff, C, taps, w, b,
                       (T*)cstate, slots, q_start, ctx_len, (T*)out, nslots, mode);
    if (taps > 1 && !one_tile)
      hipLaunchKernelGGL(conv_state_kernel<T>, dim3((C + 255) / 256, nseq), dim3(256), 0, st, (const T*)proj, ld, coff, C,
                         taps, (T*)cstate, slots, q_start, ctx_len, nslots);
  })
  return hipGetLastError();
}

GRAG_API int grag_ssm_chunk() { return SSM_CHUNK; }

template <typename T, int MODE>
static hipError_t launch_ssm_scan(const T* xbc, int C, int boff, int coff, const T* proj, int ld, int dtoff,
                                  const float* dt_bias, const float* A_log, const float* Dv, float* state,
                                  const int* slots, const int* q_start, const int* ctx_len, float* out, int nseq, int H,
                                  int G, int N, int P, int nslots, float* ws, float* wa, int maxchunks, hipStream_t st) {
  const int threads = ((P + 63) / 64) * 64;
  const size_t bytes = ((size_t)16 * (2 * ((N + 3) & ~3) + P) + 32) * sizeof(float);
  const dim3 grid(H, nseq, MODE == 0 ? 1 : maxchunks);
#define SSM_LAUNCH(NM)                                                                                              \
  hipLaunchKernelGGL((ssm_scan_kernel<T, NM, MODE>), grid, dim3(threads), bytes, st, xbc, C, boff, coff, proj, ld,  \
                     dtoff, dt_bias, A_log, Dv, state, slots, q_start, ctx_len, out, H, G, N, P, nslots, ws, wa,    \
                     maxchunks)
  if (N <= 16) {
    SSM_LAUNCH(16);
  } else if (N <= 32) {
    SSM_LAUNCH(32);
  } else if (N <= 64) {
    SSM_LAUNCH(64);
  } else if (N <= 128) {
    SSM_LAUNCH(128);
  } else {
    SSM_LAUNCH(256);
  }
#undef SSM_LAUNCH
  return hipGetLastError();
}

// ws / wa: null (or max_q_len <= the chunk length) -> one workgroup per (sequence, head) walks the whole portion; else
// the chunk-parallel passes over ws [nseq * ceil(max_q_len / chunk), H, N, P] and wa [nseq * chunks, H] fp32.
GRAG_API hipError_t grag_ssm_scan(const void* xbc, int C, int boff, int coff, const void* proj, int ld, int dtoff,
                                  const float* dt_bias, const float* A_log, const float* Dv, float* state,
                                  const int* slots, const int* q_start, const int* ctx_len, float* out, int nseq, int H,
                                  int G, int N, int P, int nslots, int dt, float* ws, float* wa, int max_q_len,
                                  hipStream_t st) {
  if (nseq <= 0) return hipSuccess;
  if (N > 256 || P > 256 || N < 1 || P < 1 || G < 1 || H % G || nseq > 65535) return hipErrorInvalidValue;
  if (ws == nullptr || wa == nullptr || max_q_len <= SSM_CHUNK) {
    DT_DISPATCH(dt, return (launch_ssm_scan<T, 0>((const T*)xbc, C, boff, coff, (const T*)proj, ld, dtoff, dt_bias, A_log,
                                                  Dv, state, slots, q_start, ctx_len, out, nseq, H, G, N, P, nslots,
                                                  nullptr, nullptr, 0, st));)
  }
  const int maxchunks = (max_q_len + SSM_CHUNK - 1) / SSM_CHUNK;
  if (maxchunks > 65535) return hipErrorInvalidValue;
  hipError_t e;
  DT_DISPATCH(dt, e = (launch_ssm_scan<T, 1>((const T*)xbc, C, boff, coff, (const T*)proj, ld, dtoff, dt_bias, A_log, Dv,
                                             state, slots, q_start, ctx_len, out, nseq, H, G, N, P, nslots, ws, wa,
                                             maxchunks, st));)
  if (e != hipSuccess) return e;
  hipLaunchKernelGGL(ssm_chunk_prefix_kernel, dim3(H, nseq, (N * P + 255) / 256), dim3(256), 0, st, state, slots,
                     q_start, ctx_len, ws, wa, maxchunks, H, N * P, nslots);
  DT_DISPATCH(dt, e = (launch_ssm_scan<T, 2>((const T*)xbc, C, boff, coff, (const T*)proj, ld, dtoff, dt_bias, A_log, Dv,
                                             state, slots, q_start, ctx_len, out, nseq, H, G, N, P, nslots, ws, wa,
                                             maxchunks, st));)
  return e;
}

GRAG_API int grag_chan_scan_tile() { return SC_CH; }
GRAG_API int grag_chan_scan_max_state() { return 256; }

template <typename T, int MODE>
static hipError_t launch_chan_scan(const T* xc, const T* low, int low_ld, const T* wdt, int R, int Rp, const float* dt_bias,
                                   const float* A, const float* Dv, const T* proj, int ld, int zoff, float* state,
                                   const int* slots, const int* q_start, const int* ctx_len, T* out, int nseq, int inner,
                                   int N, int nslots, float* ws, float* wa, int chunk_len, int maxchunks, hipStream_t st) {
  const dim3 grid((inner + SC_CH - 1) / SC_CH, nseq, MODE == 0 ? 1 : maxchunks);
#define CHAN_LAUNCH(NPT)                                                                                              \
  hipLaunchKernelGGL((chan_scan_kernel<T, NPT, MODE>), grid, dim3(256), 0, st, xc, low, low_ld, wdt, R, Rp, dt_bias,  \
                     A, Dv, proj, ld, zoff, state, slots, q_start, ctx_len, out, inner, N, nslots, ws, wa, chunk_len, \
                     maxchunks)
  if (N <= 16) {
    CHAN_LAUNCH(4);
  } else if (N <= 32) {
    CHAN_LAUNCH(8);
  } else if (N <= 64) {
    CHAN_LAUNCH(16);
  } else if (N <= 128) {
    CHAN_LAUNCH(32);
  } else {
    CHAN_LAUNCH(64);
  }
#undef CHAN_LAUNCH
  return hipGetLastError();
}

template <typename T>
static hipError_t launch_chan_step(const T* xc, const T* low, int low_ld, const T* wdt, int R, int Rp, const float* dt_bias,
                                   const float* A, const float* Dv, const T* proj, int ld, int zoff, float* state,
                                   const int* slots, const int* q_start, const int* ctx_len, T* out, int nseq, int inner,
                                   int N, int nslots, hipStream_t st) {
  const int tiles = (inner + SC_CH - 1) / SC_CH;
  int SB = SC_TB;  // sequences per workgroup: as many as leave two workgroups per CU
  while (SB > 1 && (long)tiles * ((nseq + SB - 1) / SB) < 512) SB >>= 1;
  const dim3 grid(tiles, (nseq + SB - 1) / SB);
#define CHAN_STEP(NPT, G)                                                                                              \
  hipLaunchKernelGGL((chan_step_kernel<T, NPT, G>), grid, dim3(256), 0, st, xc, low, low_ld, wdt, R, Rp, dt_bias, A,   \
                     Dv, proj, ld, zoff, state, slots, q_start, ctx_len, out, nseq, SB, inner, N, nslots)
  if (N <= 16) {
    CHAN_STEP(4, 4);
  } else if (N <= 32) {
    CHAN_STEP(8, 2);
  } else if (N <= 64) {
    CHAN_STEP(16, 1);
  } else if (N <= 128) {
    CHAN_STEP(32, 1);
  } else {
    CHAN_STEP(64, 1);
  }
#undef CHAN_STEP
  return hipGetLastError();
}

// max_q_len 1: decode rows.  chunk_len 0 (or ws / wa null, or max_q_len <= chunk_len): one pass; else the chunk-parallel passes over ws [nseq *
// ceil(max_q_len / chunk_len)][inner][N] and wa [nseq * chunks][inner] fp32, chunk_len a multiple of 16.
GRAG_API hipError_t grag_chan_scan(const void* xc, const void* low, int low_ld, const void* wdt, int R, int Rp,
                                   const float* dt_bias, const float* A, const float* Dv, const void* proj, int ld,
                                   int zoff, float* state, const int* slots, const int* q_start, const int* ctx_len,
                                   void* out, int nseq, int inner, int N, int nslots, int dt, float* ws, float* wa,
                                   int chunk_len, int max_q_len, hipStream_t st) {
  if (nseq <= 0 || max_q_len <= 0) return hipSuccess;
  if (N < 1 || N > 256 || inner < 1 || R < 1 || Rp < R || Rp % 32 || nseq > 65535 || low_ld < R + 2 * N ||
      (reinterpret_cast<uintptr_t>(A) & 15) || (reinterpret_cast<uintptr_t>(state) & 15))
    return hipErrorInvalidValue;
  if (dt == 0 && (low_ld % 8 || (reinterpret_cast<uintptr_t>(low) & 15) || (reinterpret_cast<uintptr_t>(wdt) & 15)))
    return hipErrorInvalidValue;
  if (max_q_len == 1) {
    DT_DISPATCH(dt, return (launch_chan_step<T>((const T*)xc, (const T*)low, low_ld, (const T*)wdt, R, Rp, dt_bias, A, Dv,
                                                (const T*)proj, ld, zoff, state, slots, q_start, ctx_len, (T*)out, nseq,
                                                inner, N, nslots, st));)
  }
  if (ws == nullptr || wa == nullptr || chunk_len <= 0 || max_q_len <= chunk_len) {
    DT_DISPATCH(dt, return (launch_chan_scan<T, 0>((const T*)xc, (const T*)low, low_ld, (const T*)wdt, R, Rp, dt_bias, A, Dv,
                                                   (const T*)proj, ld, zoff, state, slots, q_start, ctx_len, (T*)out, nseq,
                                                   inner, N, nslots, nullptr, nullptr, 0, 0, st));)
  }
  const int maxchunks = (max_q_len + chunk_len - 1) / chunk_len;
  if (chunk_len % SC_TB || maxchunks > 65535 || (reinterpret_cast<uintptr_t>(ws) & 15)) return hipErrorInvalidValue;
  hipError_t e;
  DT_DISPATCH(dt, e = (launch_chan_scan<T, 1>((const T*)xc, (const T*)low, low_ld, (const T*)wdt, R, Rp, dt_bias, A, Dv,
                                              (const T*)proj, ld, zoff, state, slots, q_start, ctx_len, (T*)out, nseq,
                                              inner, N, nslots, ws, wa, chunk_len, maxchunks, st));)
  if (e != hipSuccess) return e;
  hipLaunchKernelGGL(chan_chunk_prefix_kernel, dim3((unsigned)(((size_t)inner * N + 255) / 256), nseq), dim3(256), 0, st,
                     state, slots, q_start, ctx_len, A, ws, wa, chunk_len, maxchunks, inner, N, nslots);
  DT_DISPATCH(dt, e = (launch_chan_scan<T, 2>((const T*)xc, (const T*)low, low_ld, (const T*)wdt, R, Rp, dt_bias, A, Dv,
                                              (const T*)proj, ld, zoff, state, slots, q_start, ctx_len, (T*)out, nseq,
                                              inner, N, nslots, ws, wa, chunk_len, maxchunks, st));)
  return e;
}
