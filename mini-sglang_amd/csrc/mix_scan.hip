// Kernels of the looped pre-norm hybrid decoders (grouped norms, a short causal convolution in front of every sublayer,
// mixers: gated latent attention, a selective-scan state-space layer, windowed attention with a sink and normed values;
// experts that are weighted on their input), gfx950, wave = 64 lanes.  Fourth translation unit of libmsgl_mix.so; C ABI in
// include/msgl_mix.h.
//
// Precision rules (as in seqmix.hip): the residual stream, every norm, rotary angles, attention scores and weights, step
// sizes, decays and the recurrent state are fp32 in registers and in memory; tensors that feed a matrix product are stored in
// the model dtype T (bf16 or fp32).  With T = float every kernel here is true 32-bit.
//
//   norm_conv_kernel        closes a sublayer and opens the next: x' = x + mult * sum of parts (+ a vector); h = x' normed in equal
//                           groups of the row, times w; out = h + sum_j taps[., j] h[t - (n - 1) + j] (inputs before the portion from
//                           the request's state rows, inside the portion recomputed by the workgroup that needs them); the last
//                           n - 1 inputs of every request -> staging rows (msgl_mix_commit_rows moves them after the forward)
//   selective_scan_kernel   S[c, n] <- exp(dt_c A[c, n]) S[c, n] + dt_c x_c B_n;  y_c = sum_n S[c, n] C_n + D_c x_c;  out = y silu(z);
//                           a thread owns one channel's state row in registers; long portions as parallel chunks joined by
//                           selective_join_kernel
//   sink_attn_mfma_kernel   softmax attention over the last `window` keys and the first `keep` ones, with one more term exp(sink_h) in
//                           the denominator, or as the difference of two maps over the same values (normed and gated in the same
//                           launch); bf16 caches, both products on the matrix cores, fp32 online softmax; key ranges +
//                           sink_merge_kernel / diff_merge_kernel
//   sink_attn_kernel        the same in plain fp32 (fp32 caches, heads past the matrix-core instances)
//   route_sigmoid_kernel    the `top` largest router logits win, weights = sigmoid(logit)
//   scale_rows_kernel       one copy of a token's row per chosen expert, multiplied by that choice's weight
//   route_scale_kernel      logits, choice and scaled rows of a token in one launch (steps with few tokens)
//   sigmoid_gate_kernel     out = o * sigmoid(g)
//   softcap_kernel          x <- cap tanh(x / cap)
#include "mix_common.h"

namespace {

__device__ __forceinline__ float sigmoidf_(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float siluf_(float z) { return z / (1.0f + expf(-z)); }
__device__ __forceinline__ float softplusf_(float z) { return z > 20.0f ? z : log1pf(expf(z)); }
// the decay of a state element: the library's exponential in a 32-bit engine, the hardware's in a 16-bit one
__device__ __forceinline__ float decay_exp(float z, const float*) { return expf(z); }
__device__ __forceinline__ float decay_exp(float z, const bf16_t*) { return __expf(z); }
// the same split for the scan's step size and gate (once per token and channel, but inside the serial walk)
__device__ __forceinline__ float scan_softplus(float z, const float*) { return softplusf_(z); }
__device__ __forceinline__ float scan_softplus(float z, const bf16_t*) {
  return z > 20.0f ? z : (z < -15.0f ? __expf(z) : __logf(1.0f + __expf(z)));
}
__device__ __forceinline__ float scan_silu(float z, const float*) { return siluf_(z); }
__device__ __forceinline__ float scan_silu(float z, const bf16_t*) { return z * __builtin_amdgcn_rcpf(1.0f + __expf(-z)); }

// ------------------------------------------------------------------------------------------------ residual sum + grouped norm + input convolution
// A workgroup owns TB consecutive new tokens of ONE request (cu_q given) or TB consecutive rows (cu_q null: no convolution over
// time, n = 1).  It walks them in order and keeps the last n normed rows in LDS; a thread owns the columns c = tid + 256 k of
// every row, so the rows of the ring are private to it and only the group statistics need the workgroup.  Rows before the
// workgroup's first token: inside the portion they are recomputed (same arithmetic, same order: bit-equal to what their own
// workgroup stores), before the portion they are the request's state rows (state[slot][s] = the normed row at position start -
// (n - 1) + s), before position 0 they are zero.  The workgroup that holds a request's last new token leaves the request's
// new state rows in staging[b]; the state itself is replaced after the forward, because first and last tokens of a portion run
// concurrently.
template <typename T>
__global__ __launch_bounds__(256) void norm_conv_kernel(const float* __restrict__ x_in, float* __restrict__ x_out, const T* __restrict__ y0,
                                                        int p0, const T* __restrict__ y1, int p1, float mult, const float* __restrict__ add,
                                                        const T* __restrict__ w, int groups, float eps, const T* __restrict__ taps, int n,
                                                        const float* __restrict__ state, float* __restrict__ staging, T* __restrict__ h_out,
                                                        const int* __restrict__ cu_q, const int* __restrict__ seq_lens,
                                                        const int* __restrict__ slots, int B, int rows, int W, int TB) {
  extern __shared__ float lds[];
  float* ring = lds;                       // [n][W]
  float* inv = lds + (size_t)n * W;        // [groups]
  __shared__ int s_req, s_tok0, s_cnt[256];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  int b = 0, tok_first = 0, q_len = rows, start = 0, tl0 = blockIdx.x * TB;
  if (cu_q) {
    find_group(cu_q, B, TB, s_cnt, &s_req, &s_tok0);
    b = s_req;
    if (b < 0) return;
    tok_first = cu_q[b];
    q_len = cu_q[b + 1] - tok_first;
    start = seq_lens[b] - q_len;
    tl0 = s_tok0;
  }
  const int gw = W / groups;
  const int i_begin = -(n - 1);
  const size_t slot = cu_q && n > 1 ? (size_t)slots[b] : 0;
  for (int i = i_begin; i < TB; ++i) {
    const int tl = tl0 + i;
    if (tl >= q_len) break;
    float* cur = ring + (size_t)((i - i_begin) % n) * W;
    if (tl < 0) {  // before the portion: the request's state rows (zero before the sequence)
      const bool have = start + tl >= 0;
      const float* src = state + (slot * (n - 1) + (size_t)(n - 1 + tl)) * W;
      for (int c = tid; c < W; c += 256) cur[c] = have ? src[c] : 0.f;
      continue;
    }
    const size_t t = (size_t)tok_first + tl;
    for (int c = tid; c < W; c += 256) {
      float acc = 0.f;
      for (int p = 0; p < p0; ++p) acc += ld(y0 + (t * p0 + p) * W + c);
      for (int p = 0; p < p1; ++p) acc += ld(y1 + (t * p1 + p) * W + c);
      float s = x_in[t * W + c];
      if (p0 + p1 > 0) s = fmaf(mult, acc, s);
      if (add) s += add[c];
      if (i >= 0 && x_out) x_out[t * W + c] = s;
      cur[c] = s;
    }
    __syncthreads();
    for (int g = wave; g < groups; g += 4) {
      float ss = 0.f;
      for (int k = lane; k < gw; k += 64) ss = fmaf(cur[g * gw + k], cur[g * gw + k], ss);
      ss = wave_sum(ss);
      if (lane == 0) inv[g] = 1.0f / sqrtf(ss / (float)gw + eps);
    }
    __syncthreads();
    for (int c = tid; c < W; c += 256) {
      const float h = cur[c] * inv[c / gw] * ld(w + c);
      cur[c] = h;
      if (i < 0) continue;
      float o = h;
      if (taps) {
        for (int j = 0; j < n; ++j) {
          const int back = n - 1 - j;
          o = fmaf(ld(taps + (size_t)c * n + j), ring[(size_t)((i - back - i_begin) % n) * W + c], o);
        }
      }
      st(h_out + t * W + c, o);
    }
    if (staging && n > 1 && tl == q_len - 1) {  // the request's new state rows: the inputs at local indices q_len - (n - 1) + s
      for (int s = 0; s < n - 1; ++s) {
        const int li = q_len - (n - 1) + s;
        const float* src = ring + (size_t)((li - tl0 - i_begin) % n) * W;
        float* dst = staging + ((size_t)b * (n - 1) + s) * W;
        for (int c = tid; c < W; c += 256) dst[c] = src[c];
      }
    }
  }
}

// The same with 16-byte accesses and the ring in registers, for rows whose width and groups are multiples of 8 and at most NT <= 4 taps:
// a thread owns NCH chunks of 8 consecutive columns (chunk j * 256 + tid), ring[NT - 1] is the current row, ring[k] the row NT - 1 - k
// tokens before; LDS only carries the chunks' sums of squares to the waves that add up a group.
template <typename T, int NCH, int NT>
__global__ __launch_bounds__(256) void norm_conv_vec_kernel(const float* __restrict__ x_in, float* __restrict__ x_out, const T* __restrict__ y0,
                                                            int p0, const T* __restrict__ y1, int p1, float mult, const float* __restrict__ add,
                                                            const T* __restrict__ w, int groups, float eps, const T* __restrict__ taps,
                                                            const float* __restrict__ state, float* __restrict__ staging,
                                                            T* __restrict__ h_out, const int* __restrict__ cu_q,
                                                            const int* __restrict__ seq_lens, const int* __restrict__ slots, int B, int rows,
                                                            int W, int TB) {
  extern __shared__ float lds[];
  const int nchunks = W >> 3;
  float* part = lds;            // [W / 8]
  float* inv = lds + nchunks;   // [groups]
  __shared__ int s_req, s_tok0, s_cnt[256];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  int b = 0, tok_first = 0, q_len = rows, start = 0, tl0 = blockIdx.x * TB;
  if (cu_q) {
    find_group(cu_q, B, TB, s_cnt, &s_req, &s_tok0);
    b = s_req;
    if (b < 0) return;
    tok_first = cu_q[b];
    q_len = cu_q[b + 1] - tok_first;
    start = seq_lens[b] - q_len;
    tl0 = s_tok0;
  }
  const int cpg = (W / groups) >> 3;  // chunks per group
  const size_t slot = cu_q && NT > 1 ? (size_t)slots[b] : 0;
  float ring[NT][NCH][8];
#pragma unroll
  for (int k = 0; k < NT; ++k)
#pragma unroll
    for (int j = 0; j < NCH; ++j)
#pragma unroll
      for (int e = 0; e < 8; ++e) ring[k][j][e] = 0.f;
  for (int i = -(NT - 1); i < TB; ++i) {
    const int tl = tl0 + i;
    if (tl >= q_len) break;
#pragma unroll
    for (int k = 0; k + 1 < NT; ++k)
#pragma unroll
      for (int j = 0; j < NCH; ++j)
#pragma unroll
        for (int e = 0; e < 8; ++e) ring[k][j][e] = ring[k + 1][j][e];
    if (tl < 0) {  // before the portion: the request's state rows (zero before the sequence)
      const bool have = start + tl >= 0;
      const float* src = state + (slot * (NT - 1) + (size_t)(NT - 1 + tl)) * W;
#pragma unroll
      for (int j = 0; j < NCH; ++j) {
        const int ch = j * 256 + tid;
        if (ch < nchunks && have) {
          read8(src + ch * 8, ring[NT - 1][j]);
        } else {
#pragma unroll
          for (int e = 0; e < 8; ++e) ring[NT - 1][j][e] = 0.f;
        }
      }
      continue;
    }
    const size_t t = (size_t)tok_first + tl;
#pragma unroll
    for (int j = 0; j < NCH; ++j) {
      const int ch = j * 256 + tid;
      if (ch >= nchunks) continue;
      const size_t c0 = (size_t)ch * 8;
      float acc[8], v[8], s[8];
#pragma unroll
      for (int e = 0; e < 8; ++e) acc[e] = 0.f;
      for (int p = 0; p < p0; ++p) {
        read8(y0 + (t * p0 + p) * W + c0, v);
#pragma unroll
        for (int e = 0; e < 8; ++e) acc[e] += v[e];
      }
      for (int p = 0; p < p1; ++p) {
        read8(y1 + (t * p1 + p) * W + c0, v);
#pragma unroll
        for (int e = 0; e < 8; ++e) acc[e] += v[e];
      }
      read8(x_in + t * W + c0, s);
      if (p0 + p1 > 0) {
#pragma unroll
        for (int e = 0; e < 8; ++e) s[e] = fmaf(mult, acc[e], s[e]);
      }
      if (add) {
        read8(add + c0, v);
#pragma unroll
        for (int e = 0; e < 8; ++e) s[e] += v[e];
      }
      if (i >= 0 && x_out) write8(x_out + t * W + c0, s);
      float ss = 0.f;
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        ss = fmaf(s[e], s[e], ss);
        ring[NT - 1][j][e] = s[e];
      }
      part[ch] = ss;
    }
    __syncthreads();
    for (int g = wave; g < groups; g += 4) {
      float ss = 0.f;
      for (int k = lane; k < cpg; k += 64) ss += part[g * cpg + k];
      ss = wave_sum(ss);
      if (lane == 0) inv[g] = 1.0f / sqrtf(ss / (float)(cpg * 8) + eps);
    }
    __syncthreads();
#pragma unroll
    for (int j = 0; j < NCH; ++j) {
      const int ch = j * 256 + tid;
      if (ch >= nchunks) continue;
      const size_t c0 = (size_t)ch * 8;
      float wv[8], o[8];
      read8(w + c0, wv);
      const float f = inv[ch / cpg];
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        ring[NT - 1][j][e] = ring[NT - 1][j][e] * f * wv[e];
        o[e] = ring[NT - 1][j][e];
      }
      if (i < 0) continue;
      if (taps) {
        float tv[NT][8];  // the chunk's taps: element c * NT + k of 8 NT consecutive numbers
#pragma unroll
        for (int k = 0; k < NT; ++k) read8(taps + c0 * NT + k * 8, tv[k]);
#pragma unroll
        for (int e = 0; e < 8; ++e)
#pragma unroll
          for (int k = 0; k < NT; ++k) o[e] = fmaf(tv[(e * NT + k) >> 3][(e * NT + k) & 7], ring[k][j][e], o[e]);
      }
      write8(h_out + t * W + c0, o);
    }
    if (staging && NT > 1 && tl == q_len - 1) {  // the request's new state rows: the rows NT - 1 .. 1 tokens back = ring[1 ..]
#pragma unroll
      for (int s = 0; s + 1 < NT; ++s)
#pragma unroll
        for (int j = 0; j < NCH; ++j) {
          const int ch = j * 256 + tid;
          if (ch < nchunks) write8(staging + ((size_t)b * (NT - 1) + s) * W + (size_t)ch * 8, ring[s + 1][j]);
        }
    }
  }
}

// ------------------------------------------------------------------------------------------------ selective scan
// Thread = channel c, its state row S[c, 0 : N] in NP registers (the tail unused).  Workgroup = 256 channels x (request or chunk).
// Per token: dt = softplus(dt_in[t, c] + dt_bias[c]);  S[n] <- exp(dt A[c, n]) S[n] + dt x[t, c] B[t, n];  y = sum_n S[n] C[t, n] +
// D[c] x[t, c];  out[t, c] = y silu(z[t, c]).  B and C of up to 16 tokens at a time go through LDS (every channel reads the same).
// MODE 0  a request's whole portion from its state row (zero when the portion starts at position 0), state row written back.
// Long portions are cut into chunks that run in parallel; over a chunk S_end = exp(A sum dt) S_start + L:
// MODE 1  a chunk's L (from zero) and sum dt -> scratch, no outputs (a request's last chunk is skipped: nothing follows it);
//         selective_join_kernel walks a request's chunks and leaves every chunk's start state where its L was;
// MODE 2  a chunk's outputs from its start state; the last chunk of a request writes the state row.

template <typename T, int NP, int MODE>
__global__ __launch_bounds__(256) void selective_scan_kernel(T* __restrict__ out, const T* __restrict__ x, int64_t ld_x, const T* __restrict__ z,
                                                             int64_t ld_z, const T* __restrict__ dt_in, int64_t ld_dt,
                                                             const T* __restrict__ bc, int64_t ld_bc, const float* __restrict__ A,
                                                             const float* __restrict__ dt_bias, const float* __restrict__ D,
                                                             float* __restrict__ state, const int* __restrict__ cu_q,
                                                             const int* __restrict__ seq_lens, const int* __restrict__ slots, int C, int N,
                                                             const int* __restrict__ items, const int* __restrict__ item_first,
                                                             float* __restrict__ scratch, int n_items) {
  constexpr int kScanStage = NP <= 32 ? 16 : (NP <= 64 ? 8 : 4);  // tokens staged at a time (the walk over a stage is unrolled)
  __shared__ float sB[kScanStage][NP], sC[kScanStage][NP];
  const int c = blockIdx.x * 256 + threadIdx.x;
  const bool live = c < C;
  int b, first, n_new, it = 0;
  bool last_chunk = true;
  if (MODE == 0) {
    b = blockIdx.y;
    first = cu_q[b];
    n_new = cu_q[b + 1] - first;
  } else {
    it = blockIdx.y;
    b = items[3 * it];
    first = cu_q[b] + items[3 * it + 1];
    n_new = items[3 * it + 2] - items[3 * it + 1];
    last_chunk = it == item_first[b + 1] - 1;
    if (MODE == 1 && last_chunk) return;
  }
  if (n_new <= 0) return;
  const int q_len = cu_q[b + 1] - cu_q[b];
  const bool from_zero = seq_lens[b] - q_len == 0;
  float S[NP], a[NP];
  float* srow = state + ((size_t)slots[b] * C + (live ? c : 0)) * N;
  float* lrow = scratch + ((size_t)it * C + (live ? c : 0)) * N;
  const float* init = MODE == 2 ? lrow : ((MODE == 0 && !from_zero) ? srow : nullptr);
  if (N == NP && live) {  // whole rows: 16-byte loads
#pragma unroll
    for (int k = 0; k < NP; k += 4) {
      const float4 av = *reinterpret_cast<const float4*>(A + (size_t)c * N + k);
      const float4 sv = init ? *reinterpret_cast<const float4*>(init + k) : float4{0.f, 0.f, 0.f, 0.f};
      a[k] = av.x, a[k + 1] = av.y, a[k + 2] = av.z, a[k + 3] = av.w;
      S[k] = sv.x, S[k + 1] = sv.y, S[k + 2] = sv.z, S[k + 3] = sv.w;
    }
  } else {
#pragma unroll
    for (int k = 0; k < NP; ++k) {
      a[k] = (live && k < N) ? A[(size_t)c * N + k] : 0.f;
      S[k] = (live && k < N && init) ? init[k] : 0.f;
    }
  }
  const float bias = live ? dt_bias[c] : 0.f, skip = live ? D[c] : 0.f;
  float sumdt = 0.f;
  for (int t0 = 0; t0 < n_new; t0 += kScanStage) {
    const int nt = min(kScanStage, n_new - t0);
    // the stage's own inputs of this channel: all loads in flight together, not one token's at a time inside the serial walk
    float dtv[kScanStage], xv[kScanStage], zv[kScanStage];
#pragma unroll
    for (int tt = 0; tt < kScanStage; ++tt) {
      dtv[tt] = xv[tt] = zv[tt] = 0.f;
      if (tt < nt && live) {
        const size_t t = (size_t)first + t0 + tt;
        dtv[tt] = ld(dt_in + t * ld_dt + c);
        xv[tt] = ld(x + t * ld_x + c);
        if (MODE != 1) zv[tt] = ld(z + t * ld_z + c);
      }
    }
    __syncthreads();
    for (int e = threadIdx.x; e < nt * N; e += 256) {
      const int tt = e / N, k = e - tt * N;
      const T* row = bc + (size_t)(first + t0 + tt) * ld_bc;
      sB[tt][k] = ld(row + k);
      sC[tt][k] = ld(row + N + k);
    }
    __syncthreads();
    if (!live) continue;
#pragma unroll
    for (int tt = 0; tt < kScanStage; ++tt) {
      if (tt < nt) {
        const float dt = scan_softplus(dtv[tt] + bias, x);
        const float dx = dt * xv[tt];
        float y = 0.f;
#pragma unroll
        for (int k = 0; k < NP; ++k) {
          if (k < N) {
            S[k] = fmaf(decay_exp(dt * a[k], x), S[k], dx * sB[tt][k]);
            y = fmaf(S[k], sC[tt][k], y);
          }
        }
        if (MODE == 1) {
          sumdt += dt;
        } else {
          y = fmaf(skip, xv[tt], y);
          st(out + ((size_t)first + t0 + tt) * C + c, y * scan_silu(zv[tt], x));
        }
      }
    }
  }
  if (!live) return;
  float* dst = MODE == 1 ? lrow : (last_chunk ? srow : nullptr);
  if (MODE == 1) scratch[(size_t)n_items * C * N + (size_t)it * C + c] = sumdt;
  if (!dst) return;
  if (N == NP) {
#pragma unroll
    for (int k = 0; k < NP; k += 4) *reinterpret_cast<float4*>(dst + k) = float4{S[k], S[k + 1], S[k + 2], S[k + 3]};
  } else {
#pragma unroll
    for (int k = 0; k < NP; ++k)
      if (k < N) dst[k] = S[k];
  }
}

// Thread = (request, one state element e = c * N + k): start state of every chunk of the request, written over the chunk's L.
__global__ __launch_bounds__(256) void selective_join_kernel(const float* __restrict__ state, float* __restrict__ scratch,
                                                             const float* __restrict__ A, const int* __restrict__ cu_q,
                                                             const int* __restrict__ seq_lens, const int* __restrict__ slots,
                                                             const int* __restrict__ item_first, int C, int N, int n_items) {
  const int b = blockIdx.y;
  const size_t e = (size_t)blockIdx.x * 256 + threadIdx.x, CN = (size_t)C * N;
  if (e >= CN) return;
  const int i0 = item_first[b], i1 = item_first[b + 1];
  if (i1 <= i0) return;
  const bool from_zero = seq_lens[b] - (cu_q[b + 1] - cu_q[b]) == 0;
  const float a = A[e];
  float S = from_zero ? 0.f : state[(size_t)slots[b] * CN + e];
  const float* sd = scratch + (size_t)n_items * CN + e / N;
  float L = scratch[(size_t)i0 * CN + e], d = sd[(size_t)i0 * C];
  for (int it = i0; it < i1; ++it) {
    float Ln = 0.f, dn = 0.f;
    if (it + 1 < i1) {  // the next chunk's numbers are on their way while this one is joined
      Ln = scratch[(size_t)(it + 1) * CN + e];
      dn = sd[(size_t)(it + 1) * C];
    }
    scratch[(size_t)it * CN + e] = S;
    S = fmaf(expf(a * d), S, L);
    L = Ln;
    d = dn;
  }
}

// ------------------------------------------------------------------------------------------------ softmax attention with a window and a sink
// Query head h reads key/value head h / (H / G); token i sees the keys j with 0 <= i - j < window (window <= 0: every j <= i) and the
// first `keep` keys of the sequence (j < keep, j <= i);
// weights = exp(score - max) / (sum over visible keys + exp(sink[h] - max)): the sink (may be null) has no key and no value.
// MAPS = 2: a head has two query / key rows of d side by side (q [tokens, H, 2, d], key rows [G, 2, d]), each with a softmax of its own
// over the same values; with their outputs a1 and a2, o = a1 - lam a2, o / sqrt(mean(o^2) + eps) * post * sigmoid(gate) leaves the kernel.
// The visible keys of a workgroup are walked as one list: entry v is key v below `keep_eff` kept keys that lie before the window of the
// workgroup's first token, and key v + (first windowed key - keep_eff) from there on.
// A workgroup = 16 query rows (QT tokens of one request x HB query heads of ONE key/value head) x 16 lanes, one range of the
// visible keys.  splits > 1: (max, sum, unnormalised output) per range, joined by sink_merge_kernel, where the sink enters.
constexpr int kSinkRows = 16;
constexpr int kSinkMaxDv = 1024;

struct DiffOut {  // what two maps become one output row with
  const float* lam;  // one number on the device
  const void* gate;  // T, rows ld_gate apart, columns as the output's; null: no gate
  int64_t ld_gate;
  float post, eps;
};

// MC: value columns per lane, dv <= 16 MC
template <typename T, int MAPS, int MC>
__global__ __launch_bounds__(256) void sink_attn_kernel(T* __restrict__ out, int64_t ld_out, float* __restrict__ part_o,
                                                        float* __restrict__ part_ml, const float* __restrict__ q,
                                                        const T* __restrict__ k_cache, const T* __restrict__ v_cache,
                                                        const int* __restrict__ table, int64_t table_stride, const int* __restrict__ req_rows,
                                                        const int* __restrict__ seq_lens, const int* __restrict__ cu_q, int B, int total_q,
                                                        int H, int G, int d, int dv, float scale, int window, int keep,
                                                        const float* __restrict__ sink, DiffOut df, int QT, int HB, int KT, int splits) {
  extern __shared__ float lds[];
  const int dk = MAPS * d, qs = dk + 1, vs = dv + 1;
  float* sq = lds;                      // [16][MAPS d + 1]
  float* sk = sq + kSinkRows * qs;      // [KT][MAPS d + 1]
  float* sv = sk + KT * qs;             // [KT][dv + 1]
  float* sp = sv + KT * vs;             // [MAPS][16][KT]
  __shared__ int s_req, s_tok0, s_cnt[256];
  find_group(cu_q, B, QT, s_cnt, &s_req, &s_tok0);
  const int b = s_req;
  if (b < 0) return;
  const int rep = H / G, hblocks = (rep + HB - 1) / HB;
  const int kvh = blockIdx.y / hblocks, h0 = kvh * rep + (blockIdx.y % hblocks) * HB;
  const int q_len = cu_q[b + 1] - cu_q[b];
  const int start = seq_lens[b] - q_len;  // position of the request's first new token
  const int r = threadIdx.x >> 4, l = threadIdx.x & 15;
  const int tl = s_tok0 + r / HB, hh = h0 + r % HB;
  const bool valid = r < QT * HB && tl < q_len && hh < (kvh + 1) * rep;
  const int tok = cu_q[b] + (valid ? tl : s_tok0);
  const int head = valid ? hh : h0;
  const int limit = valid ? start + tl : -1;                          // last visible key
  const int lo_row = window > 0 ? max(0, limit - window + 1) : 0;     // first visible key
  const int last_tok = min(s_tok0 + QT, q_len) - 1;
  const int n_keys = start + last_tok + 1;
  const int lo_blk = window > 0 ? max(0, start + s_tok0 - window + 1) : 0;
  const int keep_eff = min(keep, lo_blk), shift = lo_blk - keep_eff, n_vis = n_keys - shift;
  const int per = ((n_vis + splits - 1) / splits + KT - 1) / KT * KT;
  const int k_begin = blockIdx.z * per, k_end = min(n_vis, k_begin + per);
  for (int i = l; i < dk; i += 16) sq[r * qs + i] = q[((size_t)tok * H + head) * dk + i];
  const int* trow = table + (size_t)req_rows[b] * table_stride;
  float o[MAPS][MC], m[MAPS], lsum[MAPS];
#pragma unroll
  for (int a = 0; a < MAPS; ++a) {
#pragma unroll
    for (int i = 0; i < MC; ++i) o[a][i] = 0.f;
    m[a] = -INFINITY;
    lsum[a] = 0.f;
  }
  const int nkd = G * dk, nvd = G * dv;
  auto key_at = [&](int v) { return v < keep_eff ? v : v + shift; };
  for (int j0 = k_begin; j0 < k_end; j0 += KT) {
    __syncthreads();
    const int nk = min(KT, k_end - j0);
    for (int e = threadIdx.x; e < nk * dk; e += 256) {
      const int j = e / dk, i = e - j * dk;
      sk[j * qs + i] = ld(k_cache + (size_t)trow[key_at(j0 + j)] * nkd + (size_t)kvh * dk + i);
    }
    for (int e = threadIdx.x; e < nk * dv; e += 256) {
      const int j = e / dv, i = e - j * dv;
      sv[j * vs + i] = ld(v_cache + (size_t)trow[key_at(j0 + j)] * nvd + (size_t)kvh * dv + i);
    }
    __syncthreads();
    float alpha[MAPS];
#pragma unroll
    for (int a = 0; a < MAPS; ++a) {
      float* spa = sp + (size_t)a * kSinkRows * KT;
      float tmax = -INFINITY;
      for (int j = l; j < KT; j += 16) {
        float s = -INFINITY;
        const int key = key_at(j0 + j);
        if (j < nk && key <= limit && (key >= lo_row || key < keep)) {
          float acc = 0.f;
          const float* qp = sq + r * qs + a * d;
          const float* kp = sk + j * qs + a * d;
          for (int i = 0; i < d; ++i) acc = fmaf(qp[i], kp[i], acc);
          s = acc * scale;
        }
        spa[r * KT + j] = s;
        tmax = fmaxf(tmax, s);
      }
#pragma unroll
      for (int x = 8; x >= 1; x >>= 1) tmax = fmaxf(tmax, __shfl_xor(tmax, x, 64));
      const float m_new = fmaxf(m[a], tmax);
      alpha[a] = m_new == -INFINITY ? 1.0f : expf(m[a] - m_new);
      float psum = 0.f;
      for (int j = l; j < KT; j += 16) {
        const float s = spa[r * KT + j];
        const float p = s == -INFINITY ? 0.f : expf(s - m_new);
        spa[r * KT + j] = p;
        psum += p;
      }
#pragma unroll
      for (int x = 8; x >= 1; x >>= 1) psum += __shfl_xor(psum, x, 64);
      lsum[a] = fmaf(lsum[a], alpha[a], psum);
      m[a] = m_new;
    }
    __syncthreads();
#pragma unroll
    for (int a = 0; a < MAPS; ++a)
#pragma unroll
      for (int i = 0; i < MC; ++i) {
        const int c = l + 16 * i;
        if (c < dv) {
          float acc = o[a][i] * alpha[a];
          for (int j = 0; j < nk; ++j) acc = fmaf(sp[(a * kSinkRows + r) * KT + j], sv[j * vs + c], acc);
          o[a][i] = acc;
        }
      }
  }
  if (MAPS == 2 && splits == 1) {
    const float f0 = 1.0f / lsum[0], f1 = df.lam[0] / lsum[MAPS - 1];  // a row that is not valid holds no sum and is not written
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < MC; ++i) {
      o[0][i] = o[0][i] * f0 - o[MAPS - 1][i] * f1;
      if (l + 16 * i < dv) ss = fmaf(o[0][i], o[0][i], ss);
    }
#pragma unroll
    for (int x = 8; x >= 1; x >>= 1) ss += __shfl_xor(ss, x, 64);
    if (!valid) return;
    const float f = df.post / sqrtf(ss / (float)dv + df.eps);
    const T* gate = cp<T>(df.gate);
#pragma unroll
    for (int i = 0; i < MC; ++i) {
      const int c = l + 16 * i;
      if (c < dv) {
        const float gz = gate ? sigmoidf_(ld(gate + (size_t)tok * df.ld_gate + (size_t)head * dv + c)) : 1.f;
        st(out + (size_t)tok * ld_out + (size_t)head * dv + c, o[0][i] * f * gz);
      }
    }
    return;
  }
  if (!valid) return;
  if (splits == 1) {
    const float sk_h = sink ? sink[head] : -INFINITY;
    const float mf = fmaxf(m[0], sk_h);
    const float em = expf(m[0] - mf);
    const float f = em / (lsum[0] * em + (sink ? expf(sk_h - mf) : 0.f));
#pragma unroll
    for (int i = 0; i < MC; ++i) {
      const int c = l + 16 * i;
      if (c < dv) st(out + (size_t)tok * ld_out + (size_t)head * dv + c, o[0][i] * f);
    }
    return;
  }
#pragma unroll
  for (int a = 0; a < MAPS; ++a) {
    const size_t row = (((size_t)blockIdx.z * total_q + tok) * H + head) * MAPS + a;
#pragma unroll
    for (int i = 0; i < MC; ++i) {
      const int c = l + 16 * i;
      if (c < dv) part_o[row * dv + c] = o[a][i];
    }
    if (l == 0) {
      part_ml[row * 2] = m[a];
      part_ml[row * 2 + 1] = lsum[a];
    }
  }
}

// The same on the matrix cores, for bf16 caches.  A workgroup = 64 query rows ((token, head) pairs of one request and ONE key/value
// head: QT tokens x HB heads) in 4 waves of 16 rows, one key range.  Keys and values come through LDS in tiles of 64 rows, row-major,
// 16-byte padded.  Per 64-key tile and wave:
//   S^T[16 keys x 16 rows] = K . Q^T     per 16-key subtile KC x v_mfma_f32_16x16x32_bf16 (Q fragments in registers, rounded to bf16 once)
//   ONE fp32 softmax step for the tile in the lane that holds the scores (a query row's 16 keys; the row's other keys sit in the
//   lanes 16, 32 and 48 further on): new maximum, rescale of the row's sum and output, weights as bf16 B operands;
//   O^T[16 v x 16 rows] += V^T . P^T     VC x v_mfma_f32_16x16x32_bf16 per 32 keys, V^T fragments read TRANSPOSED out of the row-major
//   value tile (ds_read_b64_tr_b16).  The order of a product's 32 summands is free: lane group g takes keys 4 g .. 4 g + 3 of two
//   neighbouring subtiles on both sides, which is how the scores lie in their lanes.
// The scale and log2(e) enter with Q, so that a weight is one subtraction and one exp2; a tile that every row of the workgroup sees
// whole is not masked; a wave rescales its output only when a maximum of its rows has moved.
// SPREAD (steps with at most 16 query rows per workgroup, decode): the 16 rows belong to all four waves, wave w takes the w-th 16 keys of
// every tile with a softmax state of its own, and the four states are joined through LDS at the end.
constexpr int kNKT = 64;

template <int KC, int VC, int MAPS, bool SPREAD>
__global__ __launch_bounds__(256, MAPS == 2 && KC <= 2 && VC <= 8 ? 2 : 1) void sink_attn_mfma_kernel(bf16_t* __restrict__ out, int64_t ld_out, float* __restrict__ part_o,
                                                             float* __restrict__ part_ml, const float* __restrict__ q,
                                                             const bf16_t* __restrict__ k_cache, const bf16_t* __restrict__ v_cache,
                                                             const int* __restrict__ table, int64_t table_stride,
                                                             const int* __restrict__ req_rows, const int* __restrict__ seq_lens,
                                                             const int* __restrict__ cu_q, int B, int total_q, int H, int G, int d, int dv,
                                                             float scale, int window, int keep, const float* __restrict__ sink, DiffOut df, int QT,
                                                             int HB, int splits, int kvec, int vvec) {
  constexpr int KM = KC * 32, KS = MAPS * KM + 8, VS = VC * 16 + 8;
  extern __shared__ __attribute__((aligned(16))) uint16_t smem[];
  uint16_t* sk = smem;               // [kNKT][KS]
  uint16_t* sv = smem + kNKT * KS;   // [kNKT][VS]
  __shared__ int s_req, s_tok0, s_cnt[256];
  __shared__ int s_slot[2][kNKT];
  find_group(cu_q, B, QT, s_cnt, &s_req, &s_tok0, (int)(gridDim.x - 1 - blockIdx.x));  // last tokens, with the most keys, first
  const int b = s_req;
  if (b < 0) return;
  const int rep = H / G, hblocks = (rep + HB - 1) / HB;
  const int kvh = blockIdx.y / hblocks, h0 = kvh * rep + (blockIdx.y % hblocks) * HB, z = blockIdx.z;
  const int q_len = cu_q[b + 1] - cu_q[b];
  const int start = seq_lens[b] - q_len;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int lr = lane & 15, lg = lane >> 4;
  const int r = SPREAD ? lr : wave * 16 + lr;
  const int tl = s_tok0 + r / HB, hh = h0 + r % HB;
  const bool valid = r < QT * HB && tl < q_len && hh < (kvh + 1) * rep;
  const int tok = cu_q[b] + (valid ? tl : s_tok0);
  const int head = valid ? hh : h0;
  const int limit = valid ? start + tl : -1;
  const int lo_row = window > 0 ? max(0, limit - window + 1) : 0;
  const int last_tok = min(s_tok0 + QT, q_len) - 1;
  const int n_keys = start + last_tok + 1;
  const int lo_blk = window > 0 ? max(0, start + s_tok0 - window + 1) : 0;
  const int keep_eff = min(keep, lo_blk), shift = lo_blk - keep_eff, n_vis = n_keys - shift;
  const int per = ((n_vis + splits - 1) / splits + kNKT - 1) / kNKT * kNKT;
  const int k_begin = z * per, k_end = min(n_vis, k_begin + per);
  auto key_at = [&](int v) { return v < keep_eff ? v : v + shift; };
  const bool wave_live = __builtin_amdgcn_ballot_w64(valid) != 0;
  const float scale2 = scale * 1.4426950408889634f;
  // keys up to here are seen by every row of the workgroup, and from here on the window's lower edge too
  const int all_hi = start + s_tok0, all_lo = window > 0 ? max(0, start + last_tok - window + 1) : 0;
  bf16x8_t qf[MAPS][KC];
  f32x4_t o[MAPS][VC];
  float m[MAPS], lsum[MAPS];  // the row's maximum (the same in its four lanes) and this lane's share of the row's sum
#pragma unroll
  for (int a = 0; a < MAPS; ++a) {
    const float* qrow = q + (((size_t)tok * H + head) * MAPS + a) * d;
#pragma unroll
    for (int kc = 0; kc < KC; ++kc) {
      const int k = kc * 32 + lg * 8;
      float f[8];
#pragma unroll
      for (int e = 0; e < 8; ++e) f[e] = valid && k + e < d ? qrow[k + e] * scale2 : 0.f;
      qf[a][kc] = __builtin_bit_cast(bf16x8_t, Q4{pack_bf16(f[0], f[1]), pack_bf16(f[2], f[3]), pack_bf16(f[4], f[5]), pack_bf16(f[6], f[7])});
    }
#pragma unroll
    for (int vt = 0; vt < VC; ++vt) o[a][vt] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    m[a] = -INFINITY;
    lsum[a] = 0.f;
  }
  const int* trow = table + (size_t)req_rows[b] * table_stride;
  const size_t nkd = (size_t)G * MAPS * d, nvd = (size_t)G * dv, ko = (size_t)kvh * MAPS * d, vo = (size_t)kvh * dv;
  // the next tile's rows are requested before the current tile's products: their latency hides under the MFMAs
  constexpr int KCH = MAPS * KC * 4;  // 16-byte pieces of a key row
  constexpr int NK = (kNKT * KCH + 255) / 256, NV = (kNKT * VC * 2 + 255) / 256;
  Q4 pre_k[NK], pre_v[NV];
  auto request = [&](int j0, int buf) {
#pragma unroll
    for (int u = 0; u < NK; ++u) {
      const int e = u * 256 + threadIdx.x;
      const int key = e / KCH, ch = e - key * KCH, a = ch / (KC * 4), k = (ch - a * (KC * 4)) * 8;
      pre_k[u] = Q4{0u, 0u, 0u, 0u};
      if (e < kNKT * KCH && j0 + key < k_end && k < d)
        pre_k[u] = load8(k_cache + (size_t)s_slot[buf][key] * nkd + ko + (size_t)a * d + k, d - k, kvec != 0);
    }
#pragma unroll
    for (int u = 0; u < NV; ++u) {
      const int e = u * 256 + threadIdx.x;
      const int key = e / (VC * 2), c = (e - key * (VC * 2)) * 8;
      pre_v[u] = Q4{0u, 0u, 0u, 0u};
      if (e < kNKT * VC * 2 && j0 + key < k_end && c < dv) pre_v[u] = load8(v_cache + (size_t)s_slot[buf][key] * nvd + vo + c, dv - c, vvec != 0);
    }
  };
  if (threadIdx.x < kNKT && k_begin + (int)threadIdx.x < k_end) s_slot[0][threadIdx.x] = trow[key_at(k_begin + threadIdx.x)];
  __syncthreads();
  if (k_begin < k_end) request(k_begin, 0);
  int buf = 0;
  for (int j0 = k_begin; j0 < k_end; j0 += kNKT, buf ^= 1) {
    __syncthreads();
    if (threadIdx.x < kNKT && j0 + kNKT + (int)threadIdx.x < k_end) s_slot[buf ^ 1][threadIdx.x] = trow[key_at(j0 + kNKT + threadIdx.x)];
#pragma unroll
    for (int u = 0; u < NK; ++u) {
      const int e = u * 256 + threadIdx.x;
      const int key = e / KCH, ch = e - key * KCH;
      if (e < kNKT * KCH) *reinterpret_cast<Q4*>(&sk[key * KS + ch * 8]) = pre_k[u];
    }
#pragma unroll
    for (int u = 0; u < NV; ++u) {
      const int e = u * 256 + threadIdx.x;
      const int key = e / (VC * 2), ch = e - key * (VC * 2);
      if (e < kNKT * VC * 2) *reinterpret_cast<Q4*>(&sv[key * VS + ch * 8]) = pre_v[u];
    }
    __syncthreads();
    if (j0 + kNKT < k_end) request(j0 + kNKT, buf ^ 1);
    if (!wave_live) continue;
    constexpr int NKS = SPREAD ? 1 : kNKT / 16;
    const int ks0 = SPREAD ? wave : 0;
    const bool whole = j0 + kNKT <= k_end && key_at(j0 + kNKT - 1) <= all_hi && key_at(j0) >= all_lo;
    uint2 pf[MAPS][NKS];
#pragma unroll
    for (int a = 0; a < MAPS; ++a) {
      f32x4_t sc[NKS];
      float tmax = -INFINITY;
#pragma unroll
      for (int ks = 0; ks < NKS; ++ks) {
        f32x4_t sacc{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int kc = 0; kc < KC; ++kc) {
          const bf16x8_t kf = *reinterpret_cast<const bf16x8_t*>(&sk[((ks0 + ks) * 16 + lr) * KS + a * KM + kc * 32 + lg * 8]);
          sacc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[a][kc], sacc, 0, 0, 0);
        }
        if (!whole) {
#pragma unroll
          for (int c = 0; c < 4; ++c) {
            const int v = j0 + (ks0 + ks) * 16 + 4 * lg + c, j = key_at(v);
            if (!(j <= limit && (j >= lo_row || j < keep) && v < k_end)) sacc[c] = -INFINITY;
          }
        }
        tmax = fmaxf(tmax, fmaxf(fmaxf(sacc[0], sacc[1]), fmaxf(sacc[2], sacc[3])));
        sc[ks] = sacc;
      }
      tmax = fmaxf(tmax, __shfl_xor(tmax, 16, 64));
      tmax = fmaxf(tmax, __shfl_xor(tmax, 32, 64));
      const float m_new = fmaxf(m[a], tmax);
      const float base = m_new == -INFINITY ? 0.f : m_new;  // no visible key yet: every weight below is exp2(-inf) = 0
      const float alpha = __builtin_amdgcn_exp2f(m[a] - base);
      float psum = 0.f;
#pragma unroll
      for (int ks = 0; ks < NKS; ++ks) {
        float pe[4];
#pragma unroll
        for (int c = 0; c < 4; ++c) {
          pe[c] = __builtin_amdgcn_exp2f(sc[ks][c] - base);
          psum += pe[c];
        }
        pf[a][ks] = uint2{pack_bf16(pe[0], pe[1]), pack_bf16(pe[2], pe[3])};
      }
      lsum[a] = fmaf(lsum[a], alpha, psum);
      if (__builtin_amdgcn_ballot_w64(m_new > m[a]) != 0) {
#pragma unroll
        for (int vt = 0; vt < VC; ++vt)
#pragma unroll
          for (int c = 0; c < 4; ++c) o[a][vt][c] *= alpha;
      }
      m[a] = m_new;
    }
    const uint16_t* vbase = &sv[(ks0 * 16 + 4 * lg + (lr >> 2)) * VS + 4 * (lr & 3)];
    if constexpr (SPREAD) {
#pragma unroll
      for (int vt = 0; vt < VC; ++vt) {
        const s16x4_t vf = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4_t*)(vbase + vt * 16));
#pragma unroll
        for (int a = 0; a < MAPS; ++a)
          o[a][vt] = __builtin_amdgcn_mfma_f32_16x16x16bf16_1k(vf, __builtin_bit_cast(s16x4_t, pf[a][0]), o[a][vt], 0, 0, 0);
      }
    } else {
#pragma unroll
      for (int kp = 0; kp < NKS / 2; ++kp) {
        if (j0 + kp * 32 >= k_end) break;
#pragma unroll
        for (int vt = 0; vt < VC; ++vt) {
          const s16x4_t v0 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4_t*)(vbase + kp * 32 * VS + vt * 16));
          const s16x4_t v1 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((lds_s16x4_t*)(vbase + (kp * 32 + 16) * VS + vt * 16));
          const bf16x8_t vf = __builtin_bit_cast(bf16x8_t, __builtin_shufflevector(v0, v1, 0, 1, 2, 3, 4, 5, 6, 7));
#pragma unroll
          for (int a = 0; a < MAPS; ++a) {
            const Q4 pq{pf[a][2 * kp].x, pf[a][2 * kp].y, pf[a][2 * kp + 1].x, pf[a][2 * kp + 1].y};
            o[a][vt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, __builtin_bit_cast(bf16x8_t, pq), o[a][vt], 0, 0, 0);
          }
        }
      }
    }
  }
#pragma unroll
  for (int a = 0; a < MAPS; ++a) {
    lsum[a] += __shfl_xor(lsum[a], 16, 64);
    lsum[a] += __shfl_xor(lsum[a], 32, 64);
  }
  if constexpr (SPREAD) {
    // join the four waves' states: factors from their maxima, then the outputs pairwise (waves 2, 3 onto 0, 1, then 1 onto 0)
    static_assert((size_t)2 * MAPS * VC * 4 * 64 * sizeof(float) <= (size_t)kNKT * (KS + VS) * sizeof(uint16_t), "two waves' outputs fit the tiles' LDS");
    __shared__ float s_ml[4][MAPS][2][16];
    float* so = reinterpret_cast<float*>(smem) + lane;
    if (lg == 0) {
#pragma unroll
      for (int a = 0; a < MAPS; ++a) {
        s_ml[wave][a][0][lr] = m[a];
        s_ml[wave][a][1][lr] = lsum[a];
      }
    }
    __syncthreads();  // also: every wave has read its last tile
#pragma unroll
    for (int a = 0; a < MAPS; ++a) {
      float M = -INFINITY, L = 0.f;
#pragma unroll
      for (int w = 0; w < 4; ++w) M = fmaxf(M, s_ml[w][a][0][lr]);
      const float base = M == -INFINITY ? 0.f : M;
#pragma unroll
      for (int w = 0; w < 4; ++w) L = fmaf(s_ml[w][a][1][lr], __builtin_amdgcn_exp2f(s_ml[w][a][0][lr] - base), L);
      const float f = __builtin_amdgcn_exp2f(m[a] - base);
#pragma unroll
      for (int vt = 0; vt < VC; ++vt)
#pragma unroll
        for (int c = 0; c < 4; ++c) o[a][vt][c] *= f;
      m[a] = M;
      lsum[a] = L;
    }
    auto at = [&](int part, int a, int vt, int c) { return (((part * MAPS + a) * VC + vt) * 4 + c) * 64; };
#pragma unroll
    for (int half = 2; half >= 1; half >>= 1) {
      if (wave >= half && wave < 2 * half) {
#pragma unroll
        for (int a = 0; a < MAPS; ++a)
#pragma unroll
          for (int vt = 0; vt < VC; ++vt)
#pragma unroll
            for (int c = 0; c < 4; ++c) so[at(wave - half, a, vt, c)] = o[a][vt][c];
      }
      __syncthreads();
      if (wave < half) {
#pragma unroll
        for (int a = 0; a < MAPS; ++a)
#pragma unroll
          for (int vt = 0; vt < VC; ++vt)
#pragma unroll
            for (int c = 0; c < 4; ++c) o[a][vt][c] += so[at(wave, a, vt, c)];
      }
      __syncthreads();
    }
    if (wave != 0) return;
  }
  // the maxima leave in natural units
#pragma unroll
  for (int a = 0; a < MAPS; ++a) m[a] *= 0.6931471805599453f;
  if (MAPS == 2 && splits == 1) {
    const float f0 = 1.0f / lsum[0], f1 = df.lam[0] / lsum[MAPS - 1];  // a row that is not valid holds no sum and is not written
    float ss = 0.f;
#pragma unroll
    for (int vt = 0; vt < VC; ++vt)
#pragma unroll
      for (int c = 0; c < 4; ++c) {
        o[0][vt][c] = o[0][vt][c] * f0 - o[MAPS - 1][vt][c] * f1;
        ss = fmaf(o[0][vt][c], o[0][vt][c], ss);  // columns past dv are zero
      }
    ss += __shfl_xor(ss, 16, 64);
    ss += __shfl_xor(ss, 32, 64);
    if (!valid) return;
    const float f = df.post / sqrtf(ss / (float)dv + df.eps);
    const bf16_t* gate = cp<bf16_t>(df.gate);
#pragma unroll
    for (int vt = 0; vt < VC; ++vt)
#pragma unroll
      for (int c = 0; c < 4; ++c) {
        const int v = vt * 16 + 4 * lg + c;
        if (v < dv) {
          const float gz = gate ? 1.0f / (1.0f + __expf(-ld(gate + (size_t)tok * df.ld_gate + (size_t)head * dv + v))) : 1.f;
          st(out + (size_t)tok * ld_out + (size_t)head * dv + v, o[0][vt][c] * f * gz);
        }
      }
    return;
  }
  if (!valid) return;
  if (splits == 1) {
    const float sk_h = sink ? sink[head] : -INFINITY;
    const float mf = fmaxf(m[0], sk_h);
    const float em = __expf(m[0] - mf);
    const float f = em / (lsum[0] * em + (sink ? __expf(sk_h - mf) : 0.f));
#pragma unroll
    for (int vt = 0; vt < VC; ++vt)
#pragma unroll
      for (int c = 0; c < 4; ++c) {
        const int v = vt * 16 + 4 * lg + c;
        if (v < dv) st(out + (size_t)tok * ld_out + (size_t)head * dv + v, o[0][vt][c] * f);
      }
    return;
  }
#pragma unroll
  for (int a = 0; a < MAPS; ++a) {
    const size_t row = (((size_t)z * total_q + tok) * H + head) * MAPS + a;
#pragma unroll
    for (int vt = 0; vt < VC; ++vt)
#pragma unroll
      for (int c = 0; c < 4; ++c) {
        const int v = vt * 16 + 4 * lg + c;
        if (v < dv) part_o[row * dv + v] = o[a][vt][c];
      }
    if (lg == 0) {
      part_ml[row * 2] = m[a];
      part_ml[row * 2 + 1] = lsum[a];
    }
  }
}

// One wave per (token, head): the ranges' (max, sum, output) and the sink -> the normalised output row.
template <typename T>
__global__ __launch_bounds__(64) void sink_merge_kernel(T* __restrict__ out, int64_t ld_out, const float* __restrict__ part_o,
                                                        const float* __restrict__ part_ml, int total_q, int H, int dv, int splits,
                                                        const float* __restrict__ sink) {
  const size_t t = blockIdx.x / H;
  const int h = blockIdx.x % H;
  float M = sink ? sink[h] : -INFINITY;
  for (int s = 0; s < splits; ++s) M = fmaxf(M, part_ml[(((size_t)s * total_q + t) * H + h) * 2]);
  float den = sink ? expf(sink[h] - M) : 0.f;
  for (int s = 0; s < splits; ++s) {
    const float* ml = part_ml + (((size_t)s * total_q + t) * H + h) * 2;
    den += ml[1] * expf(ml[0] - M);
  }
  for (int c = threadIdx.x; c < dv; c += 64) {
    float v = 0.f;
    for (int s = 0; s < splits; ++s)
      v = fmaf(part_o[((size_t)s * total_q + t) * H * dv + (size_t)h * dv + c], expf(part_ml[(((size_t)s * total_q + t) * H + h) * 2] - M), v);
    st(out + t * ld_out + (size_t)h * dv + c, v / den);
  }
}

// The same for two maps: both joined over the ranges, then their difference, its norm, the factor and the gate.
template <typename T>
__global__ __launch_bounds__(64) void diff_merge_kernel(T* __restrict__ out, int64_t ld_out, const float* __restrict__ part_o,
                                                        const float* __restrict__ part_ml, int total_q, int H, int dv, int splits, DiffOut df) {
  const size_t t = blockIdx.x / H;
  const int h = blockIdx.x % H;
  float M[2] = {-INFINITY, -INFINITY}, f[2];
  for (int s = 0; s < splits; ++s)
#pragma unroll
    for (int a = 0; a < 2; ++a) M[a] = fmaxf(M[a], part_ml[((((size_t)s * total_q + t) * H + h) * 2 + a) * 2]);
#pragma unroll
  for (int a = 0; a < 2; ++a) {
    float den = 0.f;
    for (int s = 0; s < splits; ++s) {
      const float* ml = part_ml + ((((size_t)s * total_q + t) * H + h) * 2 + a) * 2;
      den += ml[1] * expf(ml[0] - M[a]);
    }
    f[a] = (a == 0 ? 1.0f : -df.lam[0]) / den;
  }
  float o[kSinkMaxDv / 64], ss = 0.f;
#pragma unroll
  for (int i = 0; i < kSinkMaxDv / 64; ++i) {
    const int c = threadIdx.x + 64 * i;
    o[i] = 0.f;
    if (c < dv) {
      for (int s = 0; s < splits; ++s)
#pragma unroll
        for (int a = 0; a < 2; ++a) {
          const size_t row = (((size_t)s * total_q + t) * H + h) * 2 + a;
          o[i] = fmaf(part_o[row * dv + c], f[a] * expf(part_ml[row * 2] - M[a]), o[i]);
        }
      ss = fmaf(o[i], o[i], ss);
    }
  }
  const float n = df.post / sqrtf(wave_sum(ss) / (float)dv + df.eps);
  const T* gate = cp<T>(df.gate);
#pragma unroll
  for (int i = 0; i < kSinkMaxDv / 64; ++i) {
    const int c = threadIdx.x + 64 * i;
    if (c < dv) {
      const float gz = gate ? sigmoidf_(ld(gate + t * df.ld_gate + (size_t)h * dv + c)) : 1.f;
      st(out + t * ld_out + (size_t)h * dv + c, o[i] * n * gz);
    }
  }
}

// ------------------------------------------------------------------------------------------------ router, expert inputs, gates, cap
// z: fp32 logits [tokens, E].  The `top` largest win (ties: lowest index); the weight of a choice is sigmoid(its logit).
__global__ __launch_bounds__(64) void route_sigmoid_kernel(int* __restrict__ ids, float* __restrict__ wts, const float* __restrict__ z,
                                                           int tokens, int E, int top, int TPB) {
  extern __shared__ float lds[];
  const int t = blockIdx.x * TPB + threadIdx.x;
  if (threadIdx.x >= TPB || t >= tokens) return;
  float* s = lds + threadIdx.x;
  for (int e = 0; e < E; ++e) s[e * TPB] = z[(size_t)t * E + e];
  for (int k = 0; k < top; ++k) {
    int best = 0;
    float bv = -INFINITY;
    for (int e = 0; e < E; ++e) {
      const float v = s[e * TPB];
      if (v > bv) {
        best = e;
        bv = v;
      }
    }
    ids[(size_t)t * top + k] = best;
    wts[(size_t)t * top + k] = sigmoidf_(bv);
    s[best * TPB] = -INFINITY;
  }
}

// out[t * top + k, :] = wts[t, k] * h[t, :]
template <typename T>
__global__ __launch_bounds__(256) void scale_rows_kernel(T* __restrict__ out, const T* __restrict__ h, const float* __restrict__ wts, int top,
                                                         int W) {
  const size_t r = blockIdx.x;
  const float f = wts[r];
  const T* src = h + (r / top) * W;
  for (int c = threadIdx.x; c < W; c += 256) st(out + r * W + c, f * ld(src + c));
}

// Router logits, choice and the scaled rows of ONE token per workgroup, for steps with few tokens (every token re-reads the router
// matrix, so long batches take the product kernel for the logits instead): z[e] = router[e] . h (fp32 accumulation over the row as
// stored), the `top` largest win, out[t * top + k] = sigmoid(z[best_k]) * h[t].
template <typename T>
__global__ __launch_bounds__(256) void route_scale_kernel(int* __restrict__ ids, float* __restrict__ wts, T* __restrict__ out,
                                                          const T* __restrict__ h, const T* __restrict__ router, int E, int top, int W) {
  extern __shared__ float lds[];
  float* row = lds;       // [W]
  float* z = lds + W;     // [E]
  float* sel = z + E;     // [top]
  const size_t t = blockIdx.x;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  for (int c = tid; c < W; c += 256) row[c] = ld(h + t * W + c);
  __syncthreads();
  const bool vec = (W & 7) == 0 && ((uintptr_t)router & 15u) == 0;
  for (int e = wave; e < E; e += 4) {
    const T* r = router + (size_t)e * W;
    float acc = 0.f;
    if (vec) {  // 16-byte loads of the expert's row, several in flight
      for (int c0 = lane * 8; c0 < W; c0 += 512) {
        float wv[8];
        read8(r + c0, wv);
#pragma unroll
        for (int i = 0; i < 8; ++i) acc = fmaf(row[c0 + i], wv[i], acc);
      }
    } else {
      for (int c = lane; c < W; c += 64) acc = fmaf(row[c], ld(r + c), acc);
    }
    acc = wave_sum(acc);
    if (lane == 0) z[e] = acc;
  }
  __syncthreads();
  if (tid == 0) {
    for (int k = 0; k < top; ++k) {
      int best = 0;
      float bv = -INFINITY;
      for (int e = 0; e < E; ++e)
        if (z[e] > bv) {
          best = e;
          bv = z[e];
        }
      ids[t * top + k] = best;
      sel[k] = wts[t * top + k] = sigmoidf_(bv);
      z[best] = -INFINITY;
    }
  }
  __syncthreads();
  for (int k = 0; k < top; ++k) {
    const float f = sel[k];
    for (int c = tid; c < W; c += 256) st(out + (t * top + k) * W + c, f * row[c]);
  }
}

template <typename T>
__global__ __launch_bounds__(256) void sigmoid_gate_kernel(T* __restrict__ out, const float* __restrict__ o, const T* __restrict__ g,
                                                           int64_t ld_g, int N) {
  const size_t t = blockIdx.x;
  for (int c = threadIdx.x; c < N; c += 256) st(out + t * N + c, o[t * N + c] * sigmoidf_(ld(g + t * ld_g + c)));
}

template <typename T>
__global__ __launch_bounds__(256) void softcap_kernel(T* __restrict__ x, int64_t stride, int N, float cap, float inv_cap) {
  T* row = x + (size_t)blockIdx.x * stride;
  for (int c = blockIdx.y * 1024 + threadIdx.x; c < min(N, (int)(blockIdx.y + 1) * 1024); c += 256) st(row + c, cap * tanhf(ld(row + c) * inv_cap));
}

}  // namespace

// ================================================================================================ C ABI
int msgl_mix_norm_conv(const float* x_in, float* x_out, const void* y0, int p0, const void* y1, int p1, float mult, const float* add,
                       const void* w, int groups, float eps, const void* taps, int n, const float* state, float* staging, void* h_out,
                       const int* cu_q, const int* seq_lens, const int* slots, int batch, int rows, int W, int dtype, void* stream) {
  MIX_REQUIRE(x_in && w && h_out && dtype_ok(dtype), "norm_conv: null pointer / dtype");
  MIX_REQUIRE(rows >= 0 && W >= 1 && groups >= 1 && W % groups == 0 && n >= 1 && n <= 64 && p0 >= 0 && p1 >= 0 && (p0 == 0 || y0) &&
                  (p1 == 0 || y1),
              "norm_conv: bad sizes W %d groups %d taps %d", W, groups, n);
  MIX_REQUIRE(x_out != x_in, "norm_conv: the sum needs a buffer of its own");
  MIX_REQUIRE(n == 1 || (taps && cu_q && seq_lens && slots && state && staging && batch >= 1),
              "norm_conv: a convolution over time needs taps, the requests and their state rows");
  if (rows == 0) return MSGL_MIX_OK;
  hipStream_t s = static_cast<hipStream_t>(stream);
  auto al16 = [](const void* p) { return ((uintptr_t)p & 15u) == 0; };
  const bool vec = W % 8 == 0 && (W / groups) % 8 == 0 && W <= 8192 && n <= 4 && al16(x_in) && al16(x_out) && al16(y0) && al16(y1) && al16(add) &&
                   al16(w) && al16(taps) && al16(state) && al16(staging) && al16(h_out);
  if (vec) {
    // enough workgroups to fill the chip before a workgroup walks more tokens: a walk of TB tokens re-reads n - 1 rows
    int TB = rows / 1024;
    TB = TB < 1 ? 1 : (TB > 8 ? 8 : TB);
    const int grid = cu_q ? (rows + TB - 1) / TB + batch : (rows + TB - 1) / TB;
    const size_t lds = ((size_t)(W / 8) + groups) * sizeof(float);
    const int nch = (W + 2047) / 2048;
#define NC_LAUNCH(NCH, NT)                                                                                                              \
  DISPATCH_T(dtype, hipLaunchKernelGGL((norm_conv_vec_kernel<T, NCH, NT>), dim3(grid), dim3(256), lds, s, x_in, x_out, cp<T>(y0), p0,   \
                                       cp<T>(y1), p1, mult, add, cp<T>(w), groups, eps, cp<T>(taps), state, staging, mp<T>(h_out), cu_q, \
                                       seq_lens, slots, batch, rows, W, TB);)
#define NC_TAPS(NCH)       \
  if (n == 1) {            \
    NC_LAUNCH(NCH, 1)      \
  } else if (n == 2) {     \
    NC_LAUNCH(NCH, 2)      \
  } else if (n == 3) {     \
    NC_LAUNCH(NCH, 3)      \
  } else {                 \
    NC_LAUNCH(NCH, 4)      \
  }
    if (nch == 1) {
      NC_TAPS(1)
    } else if (nch == 2) {
      NC_TAPS(2)
    } else {
      NC_TAPS(4)
    }
#undef NC_TAPS
#undef NC_LAUNCH
    MIX_LAUNCHED("norm_conv (16-byte accesses)");
    return MSGL_MIX_OK;
  }
  int TB = rows / 512;
  TB = TB < 1 ? 1 : (TB > 16 ? 16 : TB);
  const int grid = cu_q ? (rows + TB - 1) / TB + batch : (rows + TB - 1) / TB;
  const size_t lds = ((size_t)n * W + groups) * sizeof(float);
  DISPATCH_T(dtype, MIX_REQUIRE(ensure_lds((const void*)norm_conv_kernel<T>, lds) == 0, "norm_conv: %d rows of %d do not fit LDS", n, W);
             hipLaunchKernelGGL(norm_conv_kernel<T>, dim3(grid), dim3(256), lds, s, x_in, x_out, cp<T>(y0), p0, cp<T>(y1), p1, mult, add,
                                cp<T>(w), groups, eps, cp<T>(taps), n, state, staging, mp<T>(h_out), cu_q, seq_lens, slots, batch, rows, W,
                                TB);)
  MIX_LAUNCHED("norm_conv");
  return MSGL_MIX_OK;
}

int msgl_mix_selective_scan(void* out, const void* x, int64_t ld_x, const void* z, int64_t ld_z, const void* dt_in, int64_t ld_dt,
                            const void* bc, int64_t ld_bc, const float* A, const float* dt_bias, const float* D, float* state,
                            const int* cu_q, const int* seq_lens, const int* slots, int batch, int C, int N, int dtype, int n_items,
                            const int* items, const int* item_first, float* scratch, void* stream) {
  MIX_REQUIRE(out && x && z && dt_in && bc && A && dt_bias && D && state && cu_q && seq_lens && slots && dtype_ok(dtype),
              "selective_scan: null pointer / dtype");
  MIX_REQUIRE(batch >= 0 && C >= 1 && N >= 1 && N <= 256 && ld_x >= C && ld_z >= C && ld_dt >= C && ld_bc >= 2 * N,
              "selective_scan: bad sizes C %d N %d", C, N);
  MIX_REQUIRE(n_items == 0 || (items && item_first && scratch), "selective_scan: chunks need their lists and scratch");
  if (batch == 0) return MSGL_MIX_OK;
  hipStream_t s = static_cast<hipStream_t>(stream);
  const int cb = (C + 255) / 256;
#define SCAN_CASE(NP)                                                                                                                     \
  if (N <= NP) {                                                                                                                          \
    DISPATCH_T(dtype,                                                                                                                     \
               if (n_items == 0) {                                                                                                        \
                 hipLaunchKernelGGL((selective_scan_kernel<T, NP, 0>), dim3(cb, batch), dim3(256), 0, s, mp<T>(out), cp<T>(x), ld_x,      \
                                    cp<T>(z), ld_z, cp<T>(dt_in), ld_dt, cp<T>(bc), ld_bc, A, dt_bias, D, state, cu_q, seq_lens, slots,  \
                                    C, N, items, item_first, scratch, 0);                                                                 \
               } else {                                                                                                                   \
                 hipLaunchKernelGGL((selective_scan_kernel<T, NP, 1>), dim3(cb, n_items), dim3(256), 0, s, mp<T>(out), cp<T>(x), ld_x,    \
                                    cp<T>(z), ld_z, cp<T>(dt_in), ld_dt, cp<T>(bc), ld_bc, A, dt_bias, D, state, cu_q, seq_lens, slots,  \
                                    C, N, items, item_first, scratch, n_items);                                                           \
                 hipLaunchKernelGGL(selective_join_kernel, dim3((C * N + 255) / 256, batch), dim3(256), 0, s, state, scratch, A, cu_q, seq_lens,       \
                                    slots, item_first, C, N, n_items);                                                                    \
                 hipLaunchKernelGGL((selective_scan_kernel<T, NP, 2>), dim3(cb, n_items), dim3(256), 0, s, mp<T>(out), cp<T>(x), ld_x,    \
                                    cp<T>(z), ld_z, cp<T>(dt_in), ld_dt, cp<T>(bc), ld_bc, A, dt_bias, D, state, cu_q, seq_lens, slots,  \
                                    C, N, items, item_first, scratch, n_items);                                                           \
               })                                                                                                                         \
    MIX_LAUNCHED("selective_scan");                                                                                                       \
    return MSGL_MIX_OK;                                                                                                                   \
  }
  SCAN_CASE(16)
  SCAN_CASE(32)
  SCAN_CASE(64)
  SCAN_CASE(128)
  SCAN_CASE(256)
#undef SCAN_CASE
  return MSGL_MIX_EINVAL;
}

// both forms of the attention: MAPS = 1 with an optional sink, MAPS = 2 the difference of two maps
namespace {

template <int KC, int VC, int MAPS, bool SPREAD>
int sink_mfma_launch(dim3 grid, hipStream_t s, bf16_t* out, int64_t ld_out, float* part_o, float* part_ml, const float* q, const bf16_t* k_cache,
                     const bf16_t* v_cache, const int* table, int64_t table_stride, const int* req_rows, const int* seq_lens, const int* cu_q,
                     int batch, int total_q, int H, int G, int d, int dv, float scale, int window, int keep, const float* sink, DiffOut df,
                     int QT, int HB, int splits) {
  const size_t lds = (size_t)kNKT * ((MAPS * KC * 32 + 8) + (VC * 16 + 8)) * sizeof(uint16_t);
  const int kvec = (((uintptr_t)k_cache & 15u) == 0 && d % 8 == 0) ? 1 : 0, vvec = (((uintptr_t)v_cache & 15u) == 0 && dv % 8 == 0) ? 1 : 0;
  MIX_REQUIRE(ensure_lds((const void*)sink_attn_mfma_kernel<KC, VC, MAPS, SPREAD>, lds) == 0, "sink_attn: LDS request refused");
  hipLaunchKernelGGL((sink_attn_mfma_kernel<KC, VC, MAPS, SPREAD>), grid, dim3(256), lds, s, out, ld_out, part_o, part_ml, q, k_cache, v_cache, table,
                     table_stride, req_rows, seq_lens, cu_q, batch, total_q, H, G, d, dv, scale, window, keep, sink, df, QT, HB, splits, kvec,
                     vvec);
  MIX_LAUNCHED("sink_attn (matrix cores)");
  return MSGL_MIX_OK;
}

template <typename T, int MAPS>
int sink_merge_launch(hipStream_t s, T* out, int64_t ld_out, const float* part_o, const float* part_ml, int total_q, int H, int dv, int splits,
                      const float* sink, DiffOut df) {
  if (splits <= 1) return MSGL_MIX_OK;
  if constexpr (MAPS == 1) {
    hipLaunchKernelGGL(sink_merge_kernel<T>, dim3(total_q * H), dim3(64), 0, s, out, ld_out, part_o, part_ml, total_q, H, dv, splits, sink);
  } else {
    hipLaunchKernelGGL(diff_merge_kernel<T>, dim3(total_q * H), dim3(64), 0, s, out, ld_out, part_o, part_ml, total_q, H, dv, splits, df);
  }
  MIX_LAUNCHED("sink_attn merge");
  return MSGL_MIX_OK;
}

template <int MAPS>
int sink_attn_any(void* out, int64_t ld_out, const float* q, const void* k_cache, const void* v_cache, const int* table, int64_t table_stride,
                  const int* req_rows, const int* seq_lens, const int* cu_q, int batch, int total_q, int H, int G, int d, int dv, float scale,
                  int window, int keep, const float* sink, DiffOut df, int dtype, int splits, float* workspace, hipStream_t s) {
  MIX_REQUIRE(out && q && k_cache && v_cache && table && req_rows && seq_lens && cu_q && dtype_ok(dtype), "sink_attn: null pointer / dtype");
  MIX_REQUIRE(batch >= 1 && total_q >= 0 && H >= 1 && G >= 1 && H % G == 0 && d >= 1 && dv >= 1 && dv <= kSinkMaxDv && keep >= 0 &&
                  ld_out >= (int64_t)H * dv,
              "sink_attn: bad sizes H %d G %d d %d dv %d", H, G, d, dv);
  MIX_REQUIRE(splits >= 1 && splits <= 1024 && (splits == 1 || workspace), "sink_attn: %d splits need a workspace", splits);
  if (total_q == 0) return MSGL_MIX_OK;
  const int rep = H / G;
  float* part_o = workspace;
  float* part_ml = workspace ? workspace + (size_t)splits * total_q * H * MAPS * dv : nullptr;
  if (dtype == MSGL_MIX_BF16 && d <= 256 && dv <= 256) {
    // matrix-core kernel: the smallest (KC, VC) instance that holds d <= 32 KC and dv <= 16 VC
    int HBm = 1;
    while (HBm * 2 <= rep && HBm * 2 <= 64) HBm *= 2;
    // few rows per request (decode): 16 rows per workgroup, the tiles' keys spread over its waves
    const bool spread = HBm <= 16 && total_q <= batch * (16 / HBm);
    const int QTm = (spread ? 16 : 64) / HBm, hbl = (rep + HBm - 1) / HBm;
    const int groups_m = (total_q + QTm - 1) / QTm + batch;
    MIX_REQUIRE((int64_t)G * hbl <= 65535, "sink_attn: too many heads");
    const dim3 grid(groups_m, G * hbl, splits);
#define SINK_CASE(KC, VC)                                                                                                                  \
  if (d <= KC * 32 && dv <= VC * 16) {                                                                                                     \
    const auto launch = spread ? sink_mfma_launch<KC, VC, MAPS, true> : sink_mfma_launch<KC, VC, MAPS, false>;                             \
    const int rc = launch(grid, s, mp<bf16_t>(out), ld_out, part_o, part_ml, q, cp<bf16_t>(k_cache), cp<bf16_t>(v_cache), table,           \
                          table_stride, req_rows, seq_lens, cu_q, batch, total_q, H, G, d, dv, scale, window, keep, sink, df, QTm, HBm,    \
                          splits);                                                                                                         \
    return rc ? rc : sink_merge_launch<bf16_t, MAPS>(s, mp<bf16_t>(out), ld_out, part_o, part_ml, total_q, H, dv, splits, sink, df);       \
  }
    if constexpr (MAPS == 1) {
      SINK_CASE(2, 4)
      SINK_CASE(3, 6)
      SINK_CASE(4, 8)
      SINK_CASE(6, 12)
      SINK_CASE(8, 16)
    } else {  // the values of two maps are usually twice as wide as one map's keys; maps above 128 take the plain kernel
      SINK_CASE(1, 4)
      SINK_CASE(2, 4)
      SINK_CASE(2, 8)
      SINK_CASE(4, 8)
      SINK_CASE(4, 16)
    }
#undef SINK_CASE
  }
  int HB = 1;
  while (HB * 2 <= rep && HB * 2 <= kSinkRows) HB *= 2;
  const int QT = kSinkRows / HB, hblocks = (rep + HB - 1) / HB;
  int KT = 64;
  auto need = [&](int kt) { return (size_t)((kSinkRows + kt) * (MAPS * d + 1) + kt * (dv + 1) + MAPS * kSinkRows * kt) * sizeof(float); };
  while (KT > 8 && need(KT) > 160 * 1024) KT >>= 1;
  const size_t lds = need(KT);
  MIX_REQUIRE(lds <= 160 * 1024, "sink_attn: heads of %d / %d do not fit LDS", d, dv);
  const int groups = (total_q + QT - 1) / QT + batch;  // every request may end with one partial group
  MIX_REQUIRE((int64_t)G * hblocks <= 65535, "sink_attn: too many heads");
#define SINK_PLAIN(MC)                                                                                                                       \
  DISPATCH_T(dtype, MIX_REQUIRE((ensure_lds((const void*)sink_attn_kernel<T, MAPS, MC>, lds) == 0), "sink_attn: LDS request refused");         \
             hipLaunchKernelGGL((sink_attn_kernel<T, MAPS, MC>), dim3(groups, G * hblocks, splits), dim3(256), lds, s, mp<T>(out), ld_out, part_o, \
                                part_ml, q, cp<T>(k_cache), cp<T>(v_cache), table, table_stride, req_rows, seq_lens, cu_q, batch, total_q, H,  \
                                G, d, dv, scale, window, keep, sink, df, QT, HB, KT, splits);                                                 \
             MIX_LAUNCHED("sink_attn");                                                                                                       \
             return (sink_merge_launch<T, MAPS>(s, mp<T>(out), ld_out, part_o, part_ml, total_q, H, dv, splits, sink, df));)
  if (dv <= 256) {
    SINK_PLAIN(16)
  }
  SINK_PLAIN(64)
#undef SINK_PLAIN
}

}  // namespace

int msgl_mix_sink_attn_workspace_floats(int total_q, int H, int dv, int splits) { return splits > 1 ? total_q * H * (dv + 2) * splits : 0; }

int msgl_mix_sink_attn(void* out, int64_t ld_out, const float* q, const void* k_cache, const void* v_cache, const int* table,
                       int64_t table_stride, const int* req_rows, const int* seq_lens, const int* cu_q, int batch, int total_q, int H, int G,
                       int d, int dv, float scale, int window, int keep, const float* sink, int dtype, int splits, float* workspace,
                       void* stream) {
  return sink_attn_any<1>(out, ld_out, q, k_cache, v_cache, table, table_stride, req_rows, seq_lens, cu_q, batch, total_q, H, G, d, dv, scale,
                          window, keep, sink, DiffOut{nullptr, nullptr, 0, 1.f, 0.f}, dtype, splits, workspace, static_cast<hipStream_t>(stream));
}

int msgl_mix_diff_attn(void* out, int64_t ld_out, const float* q, const void* k_cache, const void* v_cache, const int* table,
                       int64_t table_stride, const int* req_rows, const int* seq_lens, const int* cu_q, int batch, int total_q, int H, int G,
                       int d, int dv, float scale, int window, int keep, const float* lam, float post, float eps, const void* gate,
                       int64_t ld_gate, int dtype, int splits, float* workspace, void* stream) {
  MIX_REQUIRE(lam && (!gate || ld_gate >= (int64_t)H * dv), "diff_attn: no weight of the second map, or gate rows too short");
  return sink_attn_any<2>(out, ld_out, q, k_cache, v_cache, table, table_stride, req_rows, seq_lens, cu_q, batch, total_q, H, G, d, dv, scale,
                          window, keep, nullptr, DiffOut{lam, gate, ld_gate, post, eps}, dtype, splits, workspace, static_cast<hipStream_t>(stream));
}

int msgl_mix_route_sigmoid(int* ids, float* wts, const float* z, int tokens, int E, int top, void* stream) {
  MIX_REQUIRE(ids && wts && z, "route_sigmoid: null pointer");
  MIX_REQUIRE(tokens >= 0 && E >= 1 && top >= 1 && top <= E, "route_sigmoid: bad sizes E %d top %d", E, top);
  if (tokens == 0) return MSGL_MIX_OK;
  int TPB = 64;
  while (TPB > 1 && (size_t)TPB * E * sizeof(float) > 64 * 1024) TPB >>= 1;
  MIX_REQUIRE((size_t)TPB * E * sizeof(float) <= 64 * 1024, "route_sigmoid: %d experts do not fit LDS", E);
  hipLaunchKernelGGL(route_sigmoid_kernel, dim3((tokens + TPB - 1) / TPB), dim3(64), (size_t)TPB * E * sizeof(float),
                     static_cast<hipStream_t>(stream), ids, wts, z, tokens, E, top, TPB);
  MIX_LAUNCHED("route_sigmoid");
  return MSGL_MIX_OK;
}

int msgl_mix_scale_rows(void* out, const void* h, const float* wts, int tokens, int top, int W, int dtype, void* stream) {
  MIX_REQUIRE(out && h && wts && dtype_ok(dtype) && tokens >= 0 && top >= 1 && W >= 1, "scale_rows: null pointer / sizes");
  if (tokens == 0) return MSGL_MIX_OK;
  DISPATCH_T(dtype, hipLaunchKernelGGL(scale_rows_kernel<T>, dim3(tokens * top), dim3(256), 0, static_cast<hipStream_t>(stream), mp<T>(out),
                                       cp<T>(h), wts, top, W);)
  MIX_LAUNCHED("scale_rows");
  return MSGL_MIX_OK;
}

int msgl_mix_route_scale(int* ids, float* wts, void* out, const void* h, const void* router, int tokens, int E, int top, int W, int dtype,
                         void* stream) {
  MIX_REQUIRE(ids && wts && out && h && router && dtype_ok(dtype), "route_scale: null pointer / dtype");
  MIX_REQUIRE(tokens >= 0 && E >= 1 && top >= 1 && top <= E && W >= 1, "route_scale: bad sizes E %d top %d", E, top);
  if (tokens == 0) return MSGL_MIX_OK;
  const size_t lds = ((size_t)W + E + top) * sizeof(float);
  DISPATCH_T(dtype, MIX_REQUIRE(ensure_lds((const void*)route_scale_kernel<T>, lds) == 0, "route_scale: a row of %d and %d experts do not fit LDS", W, E);
             hipLaunchKernelGGL(route_scale_kernel<T>, dim3(tokens), dim3(256), lds, static_cast<hipStream_t>(stream), ids, wts, mp<T>(out),
                                cp<T>(h), cp<T>(router), E, top, W);)
  MIX_LAUNCHED("route_scale");
  return MSGL_MIX_OK;
}

int msgl_mix_sigmoid_gate(void* out, const float* o, const void* g, int64_t ld_g, int rows, int N, int dtype, void* stream) {
  MIX_REQUIRE(out && o && g && dtype_ok(dtype) && rows >= 0 && N >= 1 && ld_g >= N, "sigmoid_gate: null pointer / sizes");
  if (rows == 0) return MSGL_MIX_OK;
  DISPATCH_T(dtype, hipLaunchKernelGGL(sigmoid_gate_kernel<T>, dim3(rows), dim3(256), 0, static_cast<hipStream_t>(stream), mp<T>(out), o,
                                       cp<T>(g), ld_g, N);)
  MIX_LAUNCHED("sigmoid_gate");
  return MSGL_MIX_OK;
}

int msgl_mix_softcap(void* x, int64_t ld, int rows, int N, float cap, int dtype, void* stream) {
  MIX_REQUIRE(x && dtype_ok(dtype) && rows >= 0 && N >= 1 && ld >= N && cap > 0.f, "softcap: null pointer / sizes / cap");
  if (rows == 0) return MSGL_MIX_OK;
  DISPATCH_T(dtype, hipLaunchKernelGGL(softcap_kernel<T>, dim3(rows, (N + 1023) / 1024), dim3(256), 0, static_cast<hipStream_t>(stream), mp<T>(x), ld, N, cap,
                                       1.0f / cap);)
  MIX_LAUNCHED("softcap");
  return MSGL_MIX_OK;
}
