// Kernels of the multi-stream hybrid decoders (several residual streams joined by small mixing matrices, an element-wise squashing in
// the place of a norm, linear attention with a fixed decay per head or a decay per key channel, clamped gated feed-forwards),
// gfx950, wave = 64 lanes.  Fifth translation unit of libmsgl_mix.so; C ABI in include/msgl_mix.h.
//
// Precision rules (as in seqmix.hip): the residual streams, norms, rotary angles, decays and their logarithms and the recurrent state
// are fp32 in registers and in memory; tensors that feed a library product are stored in the model dtype T (bf16 or fp32).  With
// T = float every kernel here is true 32-bit.
//
//   stream_norm_kernel   closes a sublayer and opens the next: x'_t = sum_s mix[s, t] x_s + out[t] y;  u = sum_s read[s] x'_s;
//                        h = (tanh(alpha u) w + b) * scale.  Element-wise: one pass over the streams per sublayer
//   decay_attn_kernel    S <- diag(a) S + k v^T, o = S^T q per (request, head), a = one number per head or exp(logsigmoid(z) / tau) per
//                        key channel; pieces of 16 tokens on the fp32 matrix cores, the state in accumulator registers; the head's
//                        RMS norm and the SiLU gate in the same launch; long portions as parallel chunks joined by
//                        decay_join_kernel
//   clamp_gate_kernel    g = min(gate, limit), u = clamp(up, -limit, limit);  g sigmoid(slope g) (u + 1)
#include "mix_common.h"

namespace {

__device__ __forceinline__ float exp_(float z, const float*) { return expf(z); }
__device__ __forceinline__ float exp_(float z, const bf16_t*) { return __expf(z); }
// log sigmoid(z): never positive, exact for large |z| of either sign
__device__ __forceinline__ float log_sigmoid_(float z, const float*) { return fminf(z, 0.f) - log1pf(expf(-fabsf(z))); }
__device__ __forceinline__ float log_sigmoid_(float z, const bf16_t*) {
  const float e = __expf(-fabsf(z));
  // log(1 + e) from the hardware logarithm loses the small e of an almost closed decay (log a near 0): the series takes over there
  const float l = e < 0.03f ? e * (1.f - e * (0.5f - e * (0.33333333f - 0.25f * e))) : __logf(1.f + e);
  return fminf(z, 0.f) - l;
}

// ------------------------------------------------------------------------------------------------ residual streams + squashing norm
// Streams: fp32 [rows, s, W].  A thread owns V consecutive columns of one row in every stream, so the update may run in place.  SM >= s:
// streams held in registers.  x_in with bcast: one row [rows, W] that stands for every stream (the embedding).
template <typename T, int SM, int V>
__global__ __launch_bounds__(256) void stream_norm_kernel(const float* x_in, int bcast, const T* __restrict__ y, const float* __restrict__ mix,
                                                          const float* __restrict__ outw, float* x_out, const float* __restrict__ read,
                                                          const T* __restrict__ w, const T* __restrict__ b, const float* __restrict__ alpha,
                                                          float scale, T* __restrict__ h_out, int s, int W, uint32_t total) {
  const uint32_t gi = blockIdx.x * 256 + threadIdx.x;
  if (gi >= total) return;
  const uint32_t per_row = W / V;
  const size_t t = gi / per_row;
  const int c0 = (int)(gi - (uint32_t)t * per_row) * V;
  float x[SM][V];
  auto load = [&](const float* p, float (&f)[V]) {
    if constexpr (V == 4) {
      const float4 a = *reinterpret_cast<const float4*>(p);
      f[0] = a.x, f[1] = a.y, f[2] = a.z, f[3] = a.w;
    } else {
      f[0] = *p;
    }
  };
  auto load_t = [&](const T* p, float (&f)[V]) {
    if constexpr (V == 4 && sizeof(T) == 2) {
      const uint2 u = *reinterpret_cast<const uint2*>(p);
      f[0] = __uint_as_float(u.x << 16), f[1] = __uint_as_float(u.x & 0xffff0000u);
      f[2] = __uint_as_float(u.y << 16), f[3] = __uint_as_float(u.y & 0xffff0000u);
    } else if constexpr (V == 4) {
      const float4 a = *reinterpret_cast<const float4*>(p);
      f[0] = a.x, f[1] = a.y, f[2] = a.z, f[3] = a.w;
    } else {
      f[0] = ld(p);
    }
  };
  if (bcast) {
    load(x_in + t * W + c0, x[0]);
#pragma unroll
    for (int k = 1; k < SM; ++k)
#pragma unroll
      for (int e = 0; e < V; ++e) x[k][e] = x[0][e];
  } else {
#pragma unroll
    for (int k = 0; k < SM; ++k)
      if (k < s) load(x_in + (t * s + k) * W + c0, x[k]);
  }
  float yv[V];
  if (y) load_t(y + t * W + c0, yv);
  float u[V];
#pragma unroll
  for (int e = 0; e < V; ++e) u[e] = 0.f;
#pragma unroll
  for (int k = 0; k < SM; ++k) {
    if (k >= s) continue;
    float n[V];
    if (y) {
      const float o = outw[k];
#pragma unroll
      for (int e = 0; e < V; ++e) n[e] = o * yv[e];
#pragma unroll
      for (int j = 0; j < SM; ++j) {
        if (j >= s) continue;
        const float m = mix[j * s + k];
#pragma unroll
        for (int e = 0; e < V; ++e) n[e] = fmaf(m, x[j][e], n[e]);
      }
    } else {
#pragma unroll
      for (int e = 0; e < V; ++e) n[e] = x[k][e];
    }
    if (x_out) {
      float* p = x_out + (t * s + k) * W + c0;
      if constexpr (V == 4) {
        *reinterpret_cast<float4*>(p) = float4{n[0], n[1], n[2], n[3]};
      } else {
        *p = n[0];
      }
    }
    const float r = read ? read[k] : 1.f;
#pragma unroll
    for (int e = 0; e < V; ++e) u[e] = fmaf(r, n[e], u[e]);
  }
  if (!h_out) return;
  float wv[V], bv[V];
  load_t(w + c0, wv);
  load_t(b + c0, bv);
  const float a = alpha[0];
  T* p = h_out + t * W + c0;
  float h[V];
#pragma unroll
  for (int e = 0; e < V; ++e) h[e] = fmaf(tanhf(a * u[e]), wv[e], bv[e]) * scale;
  if constexpr (V == 4 && sizeof(T) == 2) {
    *reinterpret_cast<uint2*>(p) = uint2{bf16_bits(h[0]) | (bf16_bits(h[1]) << 16), bf16_bits(h[2]) | (bf16_bits(h[3]) << 16)};
  } else if constexpr (V == 4) {
    *reinterpret_cast<float4*>(p) = float4{h[0], h[1], h[2], h[3]};
  } else {
    st(p, h[0]);
  }
}

// ------------------------------------------------------------------------------------------------ linear attention with decays
// Workgroup = (head, request or chunk, block of 64 NS value columns), 4 waves.  Wave w owns the 16-column strips w NS .. w NS + NS - 1 of
// the head's state S [d, dv] as matrix-core accumulators: tile (dt, strip) = 16 key channels x 16 value columns, lane (g = lane / 16,
// n = lane % 16) holds rows 16 dt + 4 g + r, r = 0 .. 3, of column n.  Tokens go through in pieces of 16; every product of a piece is
// v_mfma_f32_16x16x4_f32 (fp32 in, fp32 accumulate).  A product over 16 numbers is four of these; because the ORDER of the summands is
// free, step r takes the summands 4 g + r of the four lane groups, which is the order in which accumulators hold their rows: the state
// is the B operand of q S as it lies in its registers, and the 16 x 16 scores, computed transposed (K Q^T), are the A operand of the
// product with the values as they come out.
//   scores      P^T = K Q^T (j x i), masked to j <= i, times the decay between the two tokens
//   outputs     O = P V + Q' S          Q' = q with the decay since the piece's start
//   state       S <- decay S + K'^T V   K' = k with the decay to the piece's end
// q and k of a piece go through LDS (rows of 16 DT + 4 floats: the reads above spread over all banks); values, gates and the next
// piece's numbers go straight to registers, requested before the current piece's products.
// Decays: CHANNEL false: decay[h] per head; the decay of a row enters as a factor on rows (outputs), on score elements and on the values
// of the state update.  CHANNEL true: log a = logsigmoid(z + z_bias) * inv_tau per key channel and token; with L the running sum inside the
// piece, q e^L and k e^-L carry the decays through the products as long as no channel's L falls below -kSafeLog over the piece (a bound
// the whole workgroup checks); otherwise the scores are summed pair by pair with e^(L_i - L_j) and the update uses k e^(L_end - L), so
// nothing overflows whatever the decays are.
// Rotation (CHANNEL false only): the first rd entries of q and k turn by the token's angles.
// MODE 0  a request's whole portion from its state row (zero when the portion starts at position 0), state row written back.
// Long portions are cut into chunks that run in parallel; over a chunk S_end = diag(A) S_start + U:
// MODE 1  a chunk's U from zero (and, CHANNEL, its sums of log decays) -> scratch, no outputs; a request's last chunk is skipped
//         (nothing follows it).  decay_join_kernel then walks a request's chunks and leaves every chunk's start state where U was;
// MODE 2  a chunk's outputs from its start state; the last chunk of a request writes the state row.
constexpr int kPiece = 16;
constexpr float kSafeLog = 64.f;

struct DecayArgs {
  void* out;        // T [tokens, ld_out] (normed and gated) or, with raw, fp32 [tokens, H dv]
  int64_t ld_out;
  const void *q, *k, *v, *gate;  // T, rows ld apart (column blocks of one projection)
  int64_t ld;
  const void* z;  // T, rows ld_z apart (CHANNEL)
  int64_t ld_z;
  const float *z_bias, *decay, *cos_sin;
  const int* positions;
  const void* w;  // T [dv] or null
  float* state;
  const int *cu_q, *seq_lens, *slots, *items, *item_first;
  float *scratch, *chunk_log;
  float inv_tau, q_scale, k_scale, eps;
  int rd, interleaved, H, d, dv, raw, mode;
};

template <typename T, bool CHANNEL, int DT, int NS>
__global__ __launch_bounds__(256, DT * NS <= 16 ? 2 : 1) void decay_attn_kernel(DecayArgs a) {
  constexpr int DP = DT * 16, LD = DP + 4;
  // staging: HEAD: a thread takes one (rotation) pair of entries of TP tokens; CHANNEL: one channel of TP tokens
  constexpr int kCols = CHANNEL ? DP : DP / 2, kParts = 256 / kCols, TP = kPiece / kParts;
  static_assert(kParts >= 1 && kParts * TP == kPiece, "piece does not divide over the workgroup");
  __shared__ __attribute__((aligned(16))) float sq[kPiece * LD], sk[kPiece * LD];
  __shared__ __attribute__((aligned(16))) float sL[CHANNEL ? kPiece * LD : 4], sP[CHANNEL ? kPiece * 20 : 4], sE[CHANNEL ? DP : 4];
  __shared__ float sTot[CHANNEL ? kParts * DP : 1];
  __shared__ float red[4][kPiece];
  const int h = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, g = lane >> 4, n = lane & 15;
  const int H = a.H, d = a.d, dv = a.dv, mode = a.mode;
  int b, first, n_new, it = 0;
  bool last_chunk = true;
  if (mode == 0) {
    b = blockIdx.y;
    first = a.cu_q[b];
    n_new = a.cu_q[b + 1] - first;
  } else {
    it = blockIdx.y;
    b = a.items[3 * it];
    first = a.cu_q[b] + a.items[3 * it + 1];
    n_new = a.items[3 * it + 2] - a.items[3 * it + 1];
    last_chunk = it == a.item_first[b + 1] - 1;
    if (mode == 1 && last_chunk) return;
  }
  if (n_new <= 0) return;
  const T* tag = nullptr;
  int col[NS];
  bool cok[NS];
#pragma unroll
  for (int s = 0; s < NS; ++s) {
    col[s] = blockIdx.z * 64 * NS + (wave * NS + s) * 16 + n;
    cok[s] = col[s] < dv;
  }
  f32x4_t S[DT][NS];
  {
    const bool fresh = mode == 1 || (mode == 0 && a.seq_lens[b] == n_new);
    const float* src = mode == 0 ? a.state + ((size_t)a.slots[b] * H + h) * d * dv : a.scratch + ((size_t)it * H + h) * d * dv;
#pragma unroll
    for (int dt = 0; dt < DT; ++dt)
#pragma unroll
      for (int s = 0; s < NS; ++s)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int row = dt * 16 + 4 * g + r;
          S[dt][s][r] = (!fresh && cok[s] && row < d) ? src[(size_t)row * dv + col[s]] : 0.f;
        }
  }
  // ---- what a thread stages
  const int sc = tid % kCols, part = tid / kCols;
  int ea, eb = 0, pi = 0;  // the thread's entries, and the index of its angle
  bool turn = false;
  if constexpr (CHANNEL) {
    ea = sc;
  } else {
    const int half = a.rd >> 1;
    turn = sc < half;
    pi = sc;
    if (turn) {
      ea = a.interleaved ? 2 * sc : sc;
      eb = a.interleaved ? 2 * sc + 1 : sc + half;
    } else {
      ea = a.rd + 2 * (sc - half);
      eb = ea + 1;
    }
  }
  const T* qp = cp<T>(a.q) + (size_t)h * d;
  const T* kp = cp<T>(a.k) + (size_t)h * d;
  const T* vp = cp<T>(a.v) + (size_t)h * dv;
  const T* gp = cp<T>(a.gate) + (size_t)h * dv;
  const T* zp = CHANNEL ? cp<T>(a.z) + (size_t)h * d : nullptr;
  const float zb = CHANNEL && ea < d ? a.z_bias[(size_t)h * d + ea] : 0.f;
  constexpr int NE = CHANNEL ? 1 : 2;
  float rq[TP][NE], rk[TP][NE], rx[TP][2];  // raw q, k and (cos, sin) or (z, -) of the next piece
  float rv[NS][4], rg[NS][4];
  auto request = [&](int t0) {
#pragma unroll
    for (int u = 0; u < TP; ++u) {
      const int tt = part * TP + u, tl = t0 + tt;
      const bool ok = tl < n_new;
      const size_t t = (size_t)first + (ok ? tl : 0);
      const bool oa = ok && ea < d, ob = !CHANNEL && ok && eb < d;
      rq[u][0] = (oa && mode != 1) ? ld(qp + t * a.ld + ea) : 0.f;
      rk[u][0] = oa ? ld(kp + t * a.ld + ea) : 0.f;
      if constexpr (CHANNEL) {
        rx[u][0] = oa ? ld(zp + t * a.ld_z + ea) : 0.f;
      } else {
        rq[u][1] = (ob && mode != 1) ? ld(qp + t * a.ld + eb) : 0.f;
        rk[u][1] = ob ? ld(kp + t * a.ld + eb) : 0.f;
        rx[u][0] = 1.f;
        rx[u][1] = 0.f;
        if (turn && ok) {
          const float* cs = a.cos_sin + (size_t)a.positions[t] * a.rd;
          rx[u][0] = cs[pi];
          rx[u][1] = cs[(a.rd >> 1) + pi];
        }
      }
    }
#pragma unroll
    for (int s = 0; s < NS; ++s)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int tl = t0 + 4 * g + r;
        const bool ok = cok[s] && tl < n_new;
        rv[s][r] = ok ? ld(vp + ((size_t)first + tl) * a.ld + col[s]) : 0.f;
        rg[s][r] = (ok && mode != 1 && !a.raw) ? ld(gp + ((size_t)first + tl) * a.ld + col[s]) : 0.f;
      }
  };
  const float lg = CHANNEL ? 0.f : logf(fmaxf(a.decay[h], 1e-37f));
  float fP[4], fO[4];  // HEAD: decay between token j = 4 g + r and token i = n of a piece; decay from the piece's start to token 4 g + r
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int j = 4 * g + r;
    fP[r] = CHANNEL ? 1.f : expf(lg * (float)max(n - j, 0));
    fO[r] = CHANNEL ? 1.f : expf(lg * (float)(j + 1));
  }
  float wv[NS];
#pragma unroll
  for (int s = 0; s < NS; ++s) wv[s] = (a.w && cok[s]) ? ld(cp<T>(a.w) + col[s]) : 1.f;
  float sum_log = 0.f;
  request(0);
  for (int t0 = 0; t0 < n_new; t0 += kPiece) {
    const int nt = min(kPiece, n_new - t0);
    float cv[NS][4], cg[NS][4];
#pragma unroll
    for (int s = 0; s < NS; ++s)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        cv[s][r] = rv[s][r];
        cg[s][r] = rg[s][r];
      }
    bool safe = true;
    if constexpr (CHANNEL) {
      float L[TP], run = 0.f;
#pragma unroll
      for (int u = 0; u < TP; ++u) {
        if (part * TP + u < nt && ea < d) run += log_sigmoid_(rx[u][0] + zb, tag) * a.inv_tau;
        L[u] = run;
      }
      sTot[part * DP + sc] = run;
      safe = !__syncthreads_or(run < -kSafeLog / kParts);
      float before = 0.f, total = 0.f;
#pragma unroll
      for (int p = 0; p < kParts; ++p) {
        const float v = sTot[p * DP + sc];
        before += p < part ? v : 0.f;
        total += v;
      }
      sum_log += total;
      if (part == 0) sE[sc] = exp_(total, tag);
#pragma unroll
      for (int u = 0; u < TP; ++u) {
        const int tt = part * TP + u;
        const float l = L[u] + before, q = rq[u][0] * a.q_scale, k = rk[u][0] * a.k_scale;
        sq[tt * LD + sc] = safe ? q * exp_(l, tag) : q;
        sk[tt * LD + sc] = safe ? k * exp_(-l, tag) : k;
        if (!safe) sL[tt * LD + sc] = l;
      }
    } else {
#pragma unroll
      for (int u = 0; u < TP; ++u) {
        const int tt = part * TP + u;
        const float c = rx[u][0], s = rx[u][1];
        sq[tt * LD + ea] = (rq[u][0] * c - rq[u][1] * s) * a.q_scale;
        sq[tt * LD + eb] = (rq[u][1] * c + rq[u][0] * s) * a.q_scale;
        sk[tt * LD + ea] = (rk[u][0] * c - rk[u][1] * s) * a.k_scale;
        sk[tt * LD + eb] = (rk[u][1] * c + rk[u][0] * s) * a.k_scale;
      }
    }
    __syncthreads();
    if (t0 + kPiece < n_new) request(t0 + kPiece);
    f32x4_t P{0.f, 0.f, 0.f, 0.f};
    if (CHANNEL && !safe) {  // pair by pair: thread (i, j), every exponent at most zero
      const int i = tid >> 4, j = tid & 15;
      float acc = 0.f;
      if (j <= i && mode != 1)
        for (int c = 0; c < d; ++c) acc = fmaf(sq[i * LD + c] * sk[j * LD + c], exp_(sL[i * LD + c] - sL[j * LD + c], tag), acc);
      sP[i * 20 + j] = acc;
      __syncthreads();
      // the thread's own entries now become q e^L and k e^(L_end - L)
      float total = 0.f;
#pragma unroll
      for (int p = 0; p < kParts; ++p) total += sTot[p * DP + sc];
#pragma unroll
      for (int u = 0; u < TP; ++u) {
        const int e = (part * TP + u) * LD + sc;
        const float l = sL[e];
        sq[e] *= exp_(l, tag);
        sk[e] *= exp_(total - l, tag);
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) P[r] = sP[n * 20 + 4 * g + r];
      __syncthreads();
    } else if (mode != 1) {
#pragma unroll
      for (int dt = 0; dt < DT; ++dt) {
        const f32x4_t kf = *reinterpret_cast<const f32x4_t*>(&sk[n * LD + dt * 16 + 4 * g]);
        const f32x4_t qf = *reinterpret_cast<const f32x4_t*>(&sq[n * LD + dt * 16 + 4 * g]);
#pragma unroll
        for (int r = 0; r < 4; ++r) P = __builtin_amdgcn_mfma_f32_16x16x4f32(kf[r], qf[r], P, 0, 0, 0);
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) P[r] = 4 * g + r <= n ? P[r] * fP[r] : 0.f;
    }
    f32x4_t O[NS];
#pragma unroll
    for (int s = 0; s < NS; ++s) O[s] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    if (mode != 1) {
#pragma unroll
      for (int dt = 0; dt < DT; ++dt) {
        const f32x4_t qf = *reinterpret_cast<const f32x4_t*>(&sq[n * LD + dt * 16 + 4 * g]);
#pragma unroll
        for (int r = 0; r < 4; ++r)
#pragma unroll
          for (int s = 0; s < NS; ++s) O[s] = __builtin_amdgcn_mfma_f32_16x16x4f32(qf[r], S[dt][s][r], O[s], 0, 0, 0);
      }
      if constexpr (!CHANNEL) {
#pragma unroll
        for (int s = 0; s < NS; ++s)
#pragma unroll
          for (int r = 0; r < 4; ++r) O[s][r] *= fO[r];
      }
#pragma unroll
      for (int r = 0; r < 4; ++r)
#pragma unroll
        for (int s = 0; s < NS; ++s) O[s] = __builtin_amdgcn_mfma_f32_16x16x4f32(P[r], cv[s][r], O[s], 0, 0, 0);
    }
    // ---- state
    float fS = 1.f;
    if constexpr (!CHANNEL) {
      fS = expf(lg * (float)nt);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float f = expf(lg * (float)max(nt - 1 - (4 * g + r), 0));
#pragma unroll
        for (int s = 0; s < NS; ++s) cv[s][r] *= f;
      }
    }
#pragma unroll
    for (int dt = 0; dt < DT; ++dt) {
      f32x4_t e{fS, fS, fS, fS};
      if constexpr (CHANNEL) e = *reinterpret_cast<const f32x4_t*>(&sE[dt * 16 + 4 * g]);
      if (!CHANNEL || !safe) {
#pragma unroll
        for (int s = 0; s < NS; ++s)
#pragma unroll
          for (int r = 0; r < 4; ++r) S[dt][s][r] *= e[r];
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        if (r >= nt) continue;  // no token 4 g + r in this piece
        const float kf = sk[(4 * g + r) * LD + dt * 16 + n];
#pragma unroll
        for (int s = 0; s < NS; ++s) S[dt][s] = __builtin_amdgcn_mfma_f32_16x16x4f32(kf, cv[s][r], S[dt][s], 0, 0, 0);
      }
      if (CHANNEL && safe) {
#pragma unroll
        for (int s = 0; s < NS; ++s)
#pragma unroll
          for (int r = 0; r < 4; ++r) S[dt][s][r] *= e[r];
      }
    }
    // ---- the piece's outputs: lane holds rows 4 g + r of its columns
    if (mode != 1 && !a.raw) {
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        float ss = 0.f;
#pragma unroll
        for (int s = 0; s < NS; ++s) ss = fmaf(O[s][r], O[s][r], ss);
#pragma unroll
        for (int x = 8; x >= 1; x >>= 1) ss += __shfl_xor(ss, x, 64);
        if (n == 0) red[wave][4 * g + r] = ss;
      }
    }
    __syncthreads();
    if (mode == 1) continue;
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int tl = t0 + 4 * g + r, row = 4 * g + r;
      if (tl >= n_new) continue;
      const size_t t = (size_t)first + tl;
      if (a.raw) {
#pragma unroll
        for (int s = 0; s < NS; ++s)
          if (cok[s]) static_cast<float*>(a.out)[t * a.ld_out + (size_t)h * dv + col[s]] = O[s][r];
        continue;
      }
      const float inv = 1.0f / sqrtf((((red[0][row] + red[1][row]) + red[2][row]) + red[3][row]) / (float)dv + a.eps);
#pragma unroll
      for (int s = 0; s < NS; ++s)
        if (cok[s]) {
          const float gz = cg[s][r];
          st(mp<T>(a.out) + t * a.ld_out + (size_t)h * dv + col[s], O[s][r] * inv * wv[s] * (gz / (1.0f + exp_(-gz, tag))));
        }
    }
  }
  float* dst = mode == 1 ? a.scratch + ((size_t)it * H + h) * d * dv
                         : (last_chunk ? a.state + ((size_t)a.slots[b] * H + h) * d * dv : nullptr);
  if (CHANNEL && mode == 1 && blockIdx.z == 0 && part == 0 && ea < d) a.chunk_log[((size_t)it * H + h) * d + ea] = sum_log;
  if (!dst) return;
#pragma unroll
  for (int dt = 0; dt < DT; ++dt)
#pragma unroll
    for (int s = 0; s < NS; ++s)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int row = dt * 16 + 4 * g + r;
        if (cok[s] && row < d) dst[(size_t)row * dv + col[s]] = S[dt][s][r];
      }
}

// Thread = (request, head, state element): scratch[item] holds the chunk's own contribution U on entry (nothing for a request's last
// chunk) and the state BEFORE the chunk on exit.
__global__ __launch_bounds__(256) void decay_join_kernel(const float* __restrict__ state, float* __restrict__ scratch,
                                                         const float* __restrict__ chunk_log, const float* __restrict__ decay,
                                                         const int* __restrict__ cu_q, const int* __restrict__ seq_lens,
                                                         const int* __restrict__ slots, const int* __restrict__ items,
                                                         const int* __restrict__ item_first, int H, int d, int dv) {
  const int hh = blockIdx.x, b = blockIdx.y, dd = d * dv;
  const int e = blockIdx.z * 256 + threadIdx.x;
  const int i0 = item_first[b], i1 = item_first[b + 1];
  if (e >= dd || i0 >= i1) return;
  const bool fresh = seq_lens[b] == cu_q[b + 1] - cu_q[b];
  float cur = fresh ? 0.f : state[((size_t)slots[b] * H + hh) * dd + e];
  const float lg = chunk_log ? 0.f : logf(fmaxf(decay[hh], 1e-37f));
  auto log_of = [&](int i) { return chunk_log ? chunk_log[((size_t)i * H + hh) * d + e / dv] : lg * (float)(items[3 * i + 2] - items[3 * i + 1]); };
  float U = 0.f, l = 0.f;
  if (i0 + 1 < i1) {
    U = scratch[((size_t)i0 * H + hh) * dd + e];
    l = log_of(i0);
  }
  for (int i = i0; i < i1; ++i) {
    float Un = 0.f, ln = 0.f;
    if (i + 2 < i1) {  // the next chunk's numbers are on their way while this one is joined
      Un = scratch[((size_t)(i + 1) * H + hh) * dd + e];
      ln = log_of(i + 1);
    }
    scratch[((size_t)i * H + hh) * dd + e] = cur;
    cur = fmaf(expf(l), cur, U);
    U = Un;
    l = ln;
  }
}

// ------------------------------------------------------------------------------------------------ clamped gated activation
// rows [gate: N | up: N]; a thread takes 8 consecutive columns (16-byte accesses with VEC).
template <typename T, bool VEC>
__global__ __launch_bounds__(256) void clamp_gate_kernel(T* __restrict__ out, const T* __restrict__ gu, uint32_t groups, int N, float limit,
                                                         float slope) {
  const uint32_t gi = blockIdx.x * 256 + threadIdx.x;
  if (gi >= groups) return;
  const uint32_t per_row = (N + 7) >> 3;
  const size_t row = gi / per_row;
  const int c0 = (int)(gi - (uint32_t)row * per_row) << 3, n = N - c0 < 8 ? N - c0 : 8;
  const T* src = gu + row * 2 * N + c0;
  T* dst = out + row * N + c0;
  float x[8], u[8], y[8];
  if constexpr (VEC) {
    read8(src, x);
    read8(src + N, u);
  } else {
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      x[i] = i < n ? ld(src + i) : 0.f;
      u[i] = i < n ? ld(src + N + i) : 0.f;
    }
  }
#pragma unroll
  for (int i = 0; i < 8; ++i) {
    const float gv = fminf(x[i], limit), uv = fminf(fmaxf(u[i], -limit), limit);
    y[i] = gv / (1.0f + exp_(-slope * gv, src)) * (uv + 1.0f);
  }
  if constexpr (VEC) {
    write8(dst, y);
  } else {
#pragma unroll
    for (int i = 0; i < 8; ++i)
      if (i < n) st(dst + i, y[i]);
  }
}

template <typename T, bool CHANNEL, int DT, int NS>
int decay_launch(DecayArgs a, int batch, int n_items, int col_blocks, hipStream_t s) {
  auto go = [&](int mode, int items) {
    a.mode = mode;
    hipLaunchKernelGGL((decay_attn_kernel<T, CHANNEL, DT, NS>), dim3(a.H, items, col_blocks), dim3(256), 0, s, a);
  };
  if (n_items == 0) {
    go(0, batch);
    MIX_LAUNCHED("decay_attn");
    return MSGL_MIX_OK;
  }
  go(1, n_items);
  MIX_LAUNCHED("decay_attn (chunk states)");
  hipLaunchKernelGGL(decay_join_kernel, dim3(a.H, batch, (a.d * a.dv + 255) / 256), dim3(256), 0, s, a.state, a.scratch,
                     CHANNEL ? a.chunk_log : nullptr, a.decay, a.cu_q, a.seq_lens, a.slots, a.items, a.item_first, a.H, a.d, a.dv);
  MIX_LAUNCHED("decay_attn join");
  go(2, n_items);
  MIX_LAUNCHED("decay_attn (chunk outputs)");
  return MSGL_MIX_OK;
}

template <typename T, bool CHANNEL>
int decay_pick(const DecayArgs& a, int batch, int n_items, hipStream_t s) {
#define DECAY_CASE(DT, NS) \
  if (a.d <= DT * 16 && a.dv <= 64 * NS) return decay_launch<T, CHANNEL, DT, NS>(a, batch, n_items, 1, s);
  DECAY_CASE(2, 1)
  DECAY_CASE(4, 1)
  DECAY_CASE(4, 2)
  DECAY_CASE(8, 1)
  DECAY_CASE(8, 2)
  DECAY_CASE(8, 4)
  DECAY_CASE(16, 2)
#undef DECAY_CASE
  return decay_launch<T, CHANNEL, 16, 2>(a, batch, n_items, (a.dv + 127) / 128, s);  // raw outputs only
}

}  // namespace

// ================================================================================================ C ABI
extern "C" {

int msgl_mix_stream_norm(const float* x_in, int bcast, const void* y, const float* mix, const float* out_w, float* x_out, const float* read,
                         const void* w, const void* b, const float* alpha, float scale, void* h_out, int rows, int streams, int W, int dtype,
                         void* stream) {
  MIX_REQUIRE(x_in && dtype_ok(dtype) && (x_out || h_out), "stream_norm: null pointer / dtype");
  MIX_REQUIRE(rows >= 0 && W >= 1 && streams >= 1 && streams <= 16, "stream_norm: %d streams of %d", streams, W);
  MIX_REQUIRE(!y || (mix && out_w), "stream_norm: an update needs its matrices");
  MIX_REQUIRE(!h_out || (w && b && alpha), "stream_norm: a norm needs its weights");
  MIX_REQUIRE(!(bcast && x_out == x_in), "stream_norm: one row cannot be replaced by %d streams", streams);
  if (rows == 0) return MSGL_MIX_OK;
  hipStream_t s = static_cast<hipStream_t>(stream);
  auto al16 = [](const void* p) { return ((uintptr_t)p & 15u) == 0; };
  const bool vec = W % 4 == 0 && al16(x_in) && al16(x_out) && al16(y) && al16(w) && al16(b) && al16(h_out);
  const int64_t total = (int64_t)rows * (vec ? W / 4 : W);
  MIX_REQUIRE(total <= 0x7fffffffLL, "stream_norm: %d rows of %d", rows, W);
  const dim3 grid((unsigned)((total + 255) / 256));
#define SN_GO(SM)                                                                                                                              \
  if (streams <= SM) {                                                                                                                         \
    if (vec) {                                                                                                                                 \
      DISPATCH_T(dtype, hipLaunchKernelGGL((stream_norm_kernel<T, SM, 4>), grid, dim3(256), 0, s, x_in, bcast, cp<T>(y), mix, out_w, x_out,    \
                                           read, cp<T>(w), cp<T>(b), alpha, scale, mp<T>(h_out), streams, W, (uint32_t)total);)                          \
    } else {                                                                                                                                   \
      DISPATCH_T(dtype, hipLaunchKernelGGL((stream_norm_kernel<T, SM, 1>), grid, dim3(256), 0, s, x_in, bcast, cp<T>(y), mix, out_w, x_out,    \
                                           read, cp<T>(w), cp<T>(b), alpha, scale, mp<T>(h_out), streams, W, (uint32_t)total);)                          \
    }                                                                                                                                          \
    MIX_LAUNCHED("stream_norm");                                                                                                               \
    return MSGL_MIX_OK;                                                                                                                        \
  }
  SN_GO(1)
  SN_GO(2)
  SN_GO(3)
  SN_GO(4)
  SN_GO(8)
  SN_GO(16)
#undef SN_GO
  return MSGL_MIX_EINVAL;
}

// A workgroup that owns all value columns of a head can norm and gate its output.
int msgl_mix_decay_attn_fused(int d, int dv) { return d <= 256 && (dv <= 128 || (dv <= 256 && d <= 128)) ? 1 : 0; }

int msgl_mix_decay_attn(void* out, int64_t ld_out, int raw, const void* q, const void* k, const void* v, const void* gate, int64_t ld,
                        const void* z, int64_t ld_z, const float* z_bias, float inv_tau, const float* decay, float q_scale, float k_scale,
                        const float* cos_sin, const int* positions, int rot_dims, int interleaved, const void* w, float eps, float* state,
                        const int* cu_q, const int* seq_lens, const int* slots, int batch, int H, int d, int dv, int dtype, int n_items,
                        const int* items, const int* item_first, float* scratch, void* stream) {
  MIX_REQUIRE(out && q && k && v && state && cu_q && seq_lens && slots && dtype_ok(dtype), "decay_attn: null pointer / dtype");
  MIX_REQUIRE(raw || gate, "decay_attn: the normed output needs a gate");
  MIX_REQUIRE((z != nullptr) != (decay != nullptr), "decay_attn: either one decay per head or one per key channel");
  MIX_REQUIRE(!z || (z_bias && rot_dims == 0 && ld_z >= (int64_t)H * d), "decay_attn: channel decays need their bias and take no rotation");
  MIX_REQUIRE(batch >= 0 && batch <= 65535 && H >= 1 && d >= 1 && d <= 256 && dv >= 1, "decay_attn: bad sizes H %d d %d dv %d", H, d, dv);
  MIX_REQUIRE(raw || msgl_mix_decay_attn_fused(d, dv), "decay_attn: heads of %d x %d take the raw output", d, dv);
  MIX_REQUIRE(rot_dims >= 0 && rot_dims <= d && rot_dims % 2 == 0 && (rot_dims == 0 || (cos_sin && positions)), "decay_attn: rotation of %d", rot_dims);
  MIX_REQUIRE(ld >= (int64_t)H * (d > dv ? d : dv) && ld_out >= (int64_t)H * dv, "decay_attn: rows shorter than their heads");
  MIX_REQUIRE(n_items >= 0 && n_items <= 65535 && (n_items == 0 || (items && item_first && scratch)), "decay_attn: chunks without their lists / scratch");
  if (batch == 0) return MSGL_MIX_OK;
  hipStream_t s = static_cast<hipStream_t>(stream);
  DecayArgs a{out,       ld_out,   q,        k,    v,     gate,    ld,    z,          ld_z,    z_bias,      decay, cos_sin,
              positions, w,        state,    cu_q, seq_lens, slots, items, item_first, scratch, nullptr,     inv_tau, q_scale,
              k_scale,   eps,      rot_dims, interleaved,    H,     d,     dv,         raw,     0};
  a.chunk_log = scratch ? scratch + (size_t)n_items * H * d * dv : nullptr;
  if (dtype == MSGL_MIX_BF16) return z ? decay_pick<bf16_t, true>(a, batch, n_items, s) : decay_pick<bf16_t, false>(a, batch, n_items, s);
  return z ? decay_pick<float, true>(a, batch, n_items, s) : decay_pick<float, false>(a, batch, n_items, s);
}

int msgl_mix_clamp_gate(void* out, const void* gu, int rows, int N, float limit, float slope, int dtype, void* stream) {
  MIX_REQUIRE(out && gu && rows >= 0 && N >= 1 && dtype_ok(dtype), "clamp_gate: bad arguments");
  if (rows == 0) return MSGL_MIX_OK;
  const int64_t groups = (int64_t)rows * ((N + 7) / 8);
  const bool vec = N % 8 == 0 && ((uintptr_t)gu & 15u) == 0 && ((uintptr_t)out & 15u) == 0;
  MIX_REQUIRE(groups <= 0x7fffffffLL, "clamp_gate: %d rows of %d", rows, N);
  const dim3 grid((unsigned)((groups + 255) / 256));
  hipStream_t s = static_cast<hipStream_t>(stream);
  if (vec) {
    DISPATCH_T(dtype, hipLaunchKernelGGL((clamp_gate_kernel<T, true>), grid, dim3(256), 0, s, mp<T>(out), cp<T>(gu), (uint32_t)groups, N, limit, slope);)
  } else {
    DISPATCH_T(dtype, hipLaunchKernelGGL((clamp_gate_kernel<T, false>), grid, dim3(256), 0, s, mp<T>(out), cp<T>(gu), (uint32_t)groups, N, limit, slope);)
  }
  MIX_LAUNCHED("clamp_gate");
  return MSGL_MIX_OK;
}

}  // extern "C"
