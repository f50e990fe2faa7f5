// Kernels of the decoders that norm every sublayer's input AND its output ("sandwich" residuals): x <- x + N(f(N(x) w)) w', with the
// norm centred (mean taken off) or not; gfx950, wave = 64 lanes.  Sixth translation unit of libmsgl_mix.so; C ABI in include/msgl_mix.h.
//
// Precision rules (as in seqmix.hip): the residual stream, every norm and the router are fp32 in registers and in memory; tensors that
// feed a matrix product are stored in the model dtype T (bf16 or fp32).  With T = float every kernel here is true 32-bit.
//
//   join_norm_vec_kernel    closes a sublayer and opens the next in one pass over the row: s = weighted sum of the sublayer's outputs,
//                           x' = x + N(s) w_in, h = N(x') w_out; x may be a scaled embedding row instead; x' also leaves as a T row
//                           where a product reads the stream itself; with a router the row's experts are chosen in the same launch.
//                           Rows in registers, 16-byte accesses; one workgroup or (many rows) one wave per row
//   join_norm_kernel        the same for any width, row in LDS
//   gate_mul_kernel         act(gate) * up of rows [gate | up], act = SiLU or the tanh form of GELU
#include "mix_route.h"

namespace {

struct JoinArgs {
  const float* x_in;   // fp32 [rows, W], or null: scale * table[ids[t]]
  const void* table;   // T
  const int* ids;
  float scale;
  const void* y0;      // T [rows, p0, W], weighted by gate (fp32 [rows, p0]; null: ones)
  int p0;
  const float* gate;
  const void* y1;      // T [rows, W]
  const void* w_in;    // T [W]: norm of the sum; null: the sum as it is
  float* x_out;
  void* raw0;          // T rows ld_raw apart
  void* raw1;
  int64_t ld_raw;
  const void* w_out;   // T [W]
  void* h_out;         // T [rows, W]
  float eps;
  int centre, rows, W;
  const void* router;  // T [E, W]
  const void* bias;    // T [E]
  int E, top, G, keep;
  RouteRule rule;
  int* pick;           // [rows, top]
  float* wts;
};

// The row's numbers v[j][e] (columns 8 (j * TPR + lane) + e, where they exist) become (v - mean) / sqrt(variance + eps) * w, added to
// `onto` when that is given.  The variance is taken from the deviations, not from the squares' mean.
template <typename T, int NCH, int TPR, typename Reduce>
__device__ __forceinline__ void norm_row(float (&v)[NCH][8], const T* __restrict__ w, int nch, int lane, int W, int centre, float eps, Reduce reduce) {
  float mean = 0.f;
  if (centre) {
    float s = 0.f;
#pragma unroll
    for (int j = 0; j < NCH; ++j)
      if (j * TPR + lane < nch)
#pragma unroll
        for (int e = 0; e < 8; ++e) s += v[j][e];
    mean = reduce(s) / (float)W;
  }
  float ss = 0.f;
#pragma unroll
  for (int j = 0; j < NCH; ++j)
    if (j * TPR + lane < nch)
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        v[j][e] -= mean;
        ss = fmaf(v[j][e], v[j][e], ss);
      }
  const float inv = 1.0f / sqrtf(reduce(ss) / (float)W + eps);
#pragma unroll
  for (int j = 0; j < NCH; ++j) {
    const int ch = j * TPR + lane;
    if (ch < nch) {
      float wv[8];
      read8(w + (size_t)ch * 8, wv);
#pragma unroll
      for (int e = 0; e < 8; ++e) v[j][e] *= inv * wv[e];
    }
  }
}

// TPR threads per row: 64 (a wave), 256, or, for a routed row, 1024 (the row itself needs W / 8 of them, its router all)
template <typename T, int NCH, int TPR, bool ROUTE>
__global__ __launch_bounds__(TPR == 64 ? 256 : TPR) void join_norm_vec_kernel(JoinArgs a) {
  static_assert(!ROUTE || TPR == 1024, "a routed row has a large workgroup of its own");
  extern __shared__ float lds[];  // 16 floats; with ROUTE W + 2 E + G + top more
  const int lane = TPR == 64 ? threadIdx.x & 63 : threadIdx.x;
  const int t = TPR == 64 ? blockIdx.x * 4 + (threadIdx.x >> 6) : blockIdx.x;
  if (t >= a.rows) return;  // whole waves, and no barrier below, when TPR = 64; never otherwise
  auto reduce = [&](float v) {
    if constexpr (TPR == 64)
      return wave_sum(v);
    else if constexpr (TPR == 256)
      return block_sum256(v, lds);
    else {
      v = wave_sum(v);
      __syncthreads();
      if ((threadIdx.x & 63) == 0) lds[threadIdx.x >> 6] = v;
      __syncthreads();
      float s = 0.f;
#pragma unroll
      for (int w = 0; w < TPR / 64; ++w) s += lds[w];
      return s;
    }
  };
  const int W = a.W, nch = W >> 3;
  float x[NCH][8];
#pragma unroll
  for (int j = 0; j < NCH; ++j) {
    const int ch = j * TPR + lane;
#pragma unroll
    for (int e = 0; e < 8; ++e) x[j][e] = 0.f;
    if (ch < nch) {
      if (a.x_in) {
        read8(a.x_in + (size_t)t * W + ch * 8, x[j]);
      } else {
        read8(cp<T>(a.table) + (size_t)a.ids[t] * W + ch * 8, x[j]);
#pragma unroll
        for (int e = 0; e < 8; ++e) x[j][e] *= a.scale;
      }
    }
  }
  if (a.p0 > 0 || a.y1) {
    float s[NCH][8];
#pragma unroll
    for (int j = 0; j < NCH; ++j)
#pragma unroll
      for (int e = 0; e < 8; ++e) s[j][e] = 0.f;
#pragma unroll 2
    for (int p = 0; p < a.p0; ++p) {
      const float f = a.gate ? a.gate[(size_t)t * a.p0 + p] : 1.f;
      const T* y = cp<T>(a.y0) + ((size_t)t * a.p0 + p) * W;
#pragma unroll
      for (int j = 0; j < NCH; ++j) {
        const int ch = j * TPR + lane;
        if (ch < nch) {
          float v[8];
          read8(y + ch * 8, v);
#pragma unroll
          for (int e = 0; e < 8; ++e) s[j][e] = fmaf(f, v[e], s[j][e]);
        }
      }
    }
    if (a.y1) {
      const T* y = cp<T>(a.y1) + (size_t)t * W;
#pragma unroll
      for (int j = 0; j < NCH; ++j) {
        const int ch = j * TPR + lane;
        if (ch < nch) {
          float v[8];
          read8(y + ch * 8, v);
#pragma unroll
          for (int e = 0; e < 8; ++e) s[j][e] += v[e];
        }
      }
    }
    if (a.w_in) norm_row<T, NCH, TPR>(s, cp<T>(a.w_in), nch, lane, W, a.centre, a.eps, reduce);
#pragma unroll
    for (int j = 0; j < NCH; ++j)
#pragma unroll
      for (int e = 0; e < 8; ++e) x[j][e] += s[j][e];
  }
#pragma unroll
  for (int j = 0; j < NCH; ++j) {
    const int ch = j * TPR + lane;
    if (ch < nch) {
      if (a.x_out) write8(a.x_out + (size_t)t * W + ch * 8, x[j]);
      if (a.raw0) write8(mp<T>(a.raw0) + (size_t)t * a.ld_raw + ch * 8, x[j]);
      if (a.raw1) write8(mp<T>(a.raw1) + (size_t)t * a.ld_raw + ch * 8, x[j]);
    }
  }
  if (!a.h_out) return;
  norm_row<T, NCH, TPR>(x, cp<T>(a.w_out), nch, lane, W, a.centre, a.eps, reduce);
#pragma unroll
  for (int j = 0; j < NCH; ++j) {
    const int ch = j * TPR + lane;
    if (ch < nch) write8(mp<T>(a.h_out) + (size_t)t * W + ch * 8, x[j]);
  }
  if constexpr (ROUTE) {
    float* row = lds + 16;
    float* sc = row + W;
#pragma unroll
    for (int j = 0; j < NCH; ++j) {
      const int ch = j * TPR + lane;
      if (ch < nch) {
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          T rounded;
          st(&rounded, x[j][e]);
          row[ch * 8 + e] = ld(&rounded);
        }
      }
    }
    __syncthreads();
    router_logits<TPR / 64>(row, cp<T>(a.router), a.E, W, sc);
    __syncthreads();
    if (threadIdx.x < 64)
      select_experts_wave<T>(sc, sc + a.E, sc + 2 * a.E, cp<T>(a.bias), a.E, a.top, a.G, a.keep, a.rule, a.pick + (size_t)t * a.top,
                             a.wts + (size_t)t * a.top);
  }
}

// Any width: the row and the sum in LDS, one workgroup per row.
template <typename T>
__global__ __launch_bounds__(256) void join_norm_kernel(JoinArgs a) {
  extern __shared__ float lds[];
  float *red = lds, *x = lds + 4, *s = x + a.W;  // [4], [W], [max(W, 2 E + G + top)]
  const int t = blockIdx.x, W = a.W;
  auto norm = [&](float* v, const T* w) {  // a thread's columns are tid, tid + 256, ...: only the sums need the workgroup
    float mean = 0.f, ss = 0.f;
    if (a.centre) {
      for (int c = threadIdx.x; c < W; c += 256) mean += v[c];
      mean = block_sum256(mean, red) / (float)W;
    }
    for (int c = threadIdx.x; c < W; c += 256) {
      v[c] -= mean;
      ss = fmaf(v[c], v[c], ss);
    }
    const float inv = 1.0f / sqrtf(block_sum256(ss, red) / (float)W + a.eps);
    for (int c = threadIdx.x; c < W; c += 256) v[c] *= inv * ld(w + c);
  };
  const bool parts = a.p0 > 0 || a.y1;
  for (int c = threadIdx.x; c < W; c += 256) {
    x[c] = a.x_in ? a.x_in[(size_t)t * W + c] : a.scale * ld(cp<T>(a.table) + (size_t)a.ids[t] * W + c);
    if (!parts) continue;
    float acc = 0.f;
    for (int p = 0; p < a.p0; ++p)
      acc = fmaf(a.gate ? a.gate[(size_t)t * a.p0 + p] : 1.f, ld(cp<T>(a.y0) + ((size_t)t * a.p0 + p) * W + c), acc);
    if (a.y1) acc += ld(cp<T>(a.y1) + (size_t)t * W + c);
    s[c] = acc;
  }
  if (parts && a.w_in) norm(s, cp<T>(a.w_in));
  for (int c = threadIdx.x; c < W; c += 256) {
    if (parts) x[c] += s[c];
    if (a.x_out) a.x_out[(size_t)t * W + c] = x[c];
    if (a.raw0) st(mp<T>(a.raw0) + (size_t)t * a.ld_raw + c, x[c]);
    if (a.raw1) st(mp<T>(a.raw1) + (size_t)t * a.ld_raw + c, x[c]);
  }
  if (!a.h_out) return;
  norm(x, cp<T>(a.w_out));
  for (int c = threadIdx.x; c < W; c += 256) {
    T rounded;
    st(&rounded, x[c]);
    mp<T>(a.h_out)[(size_t)t * W + c] = rounded;
    x[c] = ld(&rounded);
  }
  if (!a.router) return;
  __syncthreads();
  router_logits<4>(x, cp<T>(a.router), a.E, W, s);
  __syncthreads();
  if (threadIdx.x < 64)
    select_experts_wave<T>(s, s + a.E, s + 2 * a.E, cp<T>(a.bias), a.E, a.top, a.G, a.keep, a.rule, a.pick + (size_t)t * a.top,
                           a.wts + (size_t)t * a.top);
}

// ------------------------------------------------------------------------------------------------ gated activation
__device__ __forceinline__ float exp_(float z, const float*) { return expf(z); }
__device__ __forceinline__ float exp_(float z, const bf16_t*) { return __expf(z); }

// z sigmoid(z), or 0.5 z (1 + tanh(u)) = z sigmoid(2 u) with u = sqrt(2 / pi) (z + 0.044715 z^3)
template <typename T, int ACT>
__device__ __forceinline__ float gate_act(float z, const T* tag) {
  if constexpr (ACT == MSGL_MIX_GATE_MUL_SILU) {
    return z / (1.0f + exp_(-z, tag));
  } else {
    const float u = 0.7978845608028654f * fmaf(0.044715f * z * z, z, z);
    return z / (1.0f + exp_(-2.0f * u, tag));
  }
}

// rows [gate: N | up: N]; a thread takes 8 consecutive columns (16-byte accesses with VEC).
template <typename T, int ACT, bool VEC>
__global__ __launch_bounds__(256) void gate_mul_kernel(T* __restrict__ out, const T* __restrict__ gu, uint32_t groups, int N) {
  const uint32_t gi = blockIdx.x * 256 + threadIdx.x;
  if (gi >= groups) return;
  const uint32_t per_row = (N + 7) >> 3;
  const size_t row = gi / per_row;
  const int c0 = (int)(gi - (uint32_t)row * per_row) << 3, n = N - c0 < 8 ? N - c0 : 8;
  const T* src = gu + row * 2 * N + c0;
  T* dst = out + row * N + c0;
  float z[8], u[8], y[8];
  if constexpr (VEC) {
    read8(src, z);
    read8(src + N, u);
  } else {
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      z[i] = i < n ? ld(src + i) : 0.f;
      u[i] = i < n ? ld(src + N + i) : 0.f;
    }
  }
#pragma unroll
  for (int i = 0; i < 8; ++i) y[i] = gate_act<T, ACT>(z[i], src) * u[i];
  if constexpr (VEC) {
    write8(dst, y);
  } else {
#pragma unroll
    for (int i = 0; i < 8; ++i)
      if (i < n) st(dst + i, y[i]);
  }
}

bool aligned16(const void* p) { return ((uintptr_t)p & 15u) == 0; }

template <typename T, int NCH, int TPR, bool ROUTE = false>
int join_launch(const JoinArgs& a, size_t lds, hipStream_t s) {
  MIX_REQUIRE(ensure_lds((const void*)join_norm_vec_kernel<T, NCH, TPR, ROUTE>, lds) == 0, "join_norm: row of %d does not fit LDS", a.W);
  hipLaunchKernelGGL((join_norm_vec_kernel<T, NCH, TPR, ROUTE>), dim3(TPR == 64 ? (a.rows + 3) / 4 : a.rows), dim3(TPR == 64 ? 256 : TPR), lds, s, a);
  MIX_LAUNCHED("join_norm");
  return MSGL_MIX_OK;
}

template <typename T>
int join_pick(const JoinArgs& a, hipStream_t s) {
  const int W = a.W;
  const size_t route = a.router ? (size_t)(2 * a.E + a.G + a.top) : 0;
  bool vec = W % 8 == 0 && a.ld_raw % 8 == 0 && W <= 256 * 8 * 4;
  for (const void* p : {(const void*)a.x_in, a.table, a.y0, a.y1, a.w_in, (const void*)a.x_out, (const void*)a.raw0, (const void*)a.raw1, a.w_out,
                        (const void*)a.h_out})
    vec = vec && aligned16(p);
  if (vec) {
    const size_t lds = (16 + (a.router ? W + route : 0)) * sizeof(float);
    if (a.router) return join_launch<T, 1, 1024, true>(a, lds, s);
    // many short rows: a wave owns a row and nothing meets at a barrier; otherwise a workgroup owns one, for more loads in flight per row
    if (a.rows >= 1024 && W <= 512) return join_launch<T, 1, 64>(a, lds, s);
    if (a.rows >= 1024 && W <= 1024) return join_launch<T, 2, 64>(a, lds, s);
    if (W <= 2048) return join_launch<T, 1, 256>(a, lds, s);
    if (W <= 4096) return join_launch<T, 2, 256>(a, lds, s);
    return join_launch<T, 4, 256>(a, lds, s);
  }
  const size_t lds = (4 + (size_t)W + ((size_t)W > route ? (size_t)W : route)) * sizeof(float);
  MIX_REQUIRE(ensure_lds((const void*)join_norm_kernel<T>, lds) == 0, "join_norm: row of %d does not fit LDS", W);
  hipLaunchKernelGGL(join_norm_kernel<T>, dim3(a.rows), dim3(256), lds, s, a);
  MIX_LAUNCHED("join_norm");
  return MSGL_MIX_OK;
}

}  // namespace

extern "C" {

int msgl_mix_join_norm(const float* x_in, const void* table, const int* ids, float scale, const void* y0, int p0, const float* gate,
                       const void* y1, const void* w_in, float* x_out, void* raw0, void* raw1, int64_t ld_raw, const void* w_out, void* h_out,
                       float eps, int centre, int rows, int W, int dtype, const void* router, const void* bias, int E, int top, int G, int keep,
                       int sigmoid, int group_best, float route_scale, int* pick, float* wts, void* stream) {
  MIX_REQUIRE(rows >= 0 && W >= 1 && dtype_ok(dtype) && ((x_in != nullptr) != (table != nullptr)) && (!table || ids),
              "join_norm: the row comes from x_in or from a table");
  MIX_REQUIRE(p0 >= 0 && (p0 == 0) == (y0 == nullptr) && (!gate || y0), "join_norm: %d weighted parts do not match y0", p0);
  MIX_REQUIRE((h_out == nullptr) == (w_out == nullptr) && (h_out || x_out || raw0 || raw1), "join_norm: nothing to write, or h without its weight");
  MIX_REQUIRE((!raw0 && !raw1) || ld_raw >= W, "join_norm: copy rows %lld apart", (long long)ld_raw);
  if (router) {
    MIX_REQUIRE(h_out && pick && wts, "join_norm: a router needs h, ids and weights");
    MIX_REQUIRE(E >= 1 && top >= 1 && top <= E && G >= 1 && E % G == 0 && keep >= 1 && keep <= G && top <= keep * (E / G),
                "join_norm: bad router sizes E %d top %d groups %d keep %d", E, top, G, keep);
    MIX_REQUIRE(group_best == 1 || group_best == 2, "join_norm: a group's score sums its 1 or 2 largest choices, not %d", group_best);
  }
  if (rows == 0) return MSGL_MIX_OK;
  const JoinArgs a{x_in, table, ids, scale, y0, p0, gate, y1, w_in, x_out, raw0, raw1, raw0 || raw1 ? ld_raw : 0, w_out, h_out, eps, centre, rows, W,
                   router, bias, E, top, G, keep, RouteRule{sigmoid, group_best, route_scale}, pick, wts};
  DISPATCH_T(dtype, return join_pick<T>(a, static_cast<hipStream_t>(stream));)
}

int msgl_mix_gate_mul(void* out, const void* gu, int rows, int N, int act, int dtype, void* stream) {
  MIX_REQUIRE(out && gu && rows >= 0 && N >= 1 && dtype_ok(dtype), "gate_mul: bad arguments");
  MIX_REQUIRE(act == MSGL_MIX_GATE_MUL_SILU || act == MSGL_MIX_GATE_MUL_GELU_TANH, "gate_mul: unknown activation %d", act);
  const int64_t groups = (int64_t)rows * ((N + 7) / 8);
  MIX_REQUIRE(groups <= 0xffffff00ll, "gate_mul: %d x %d too large", rows, N);
  if (rows == 0) return MSGL_MIX_OK;
  hipStream_t s = static_cast<hipStream_t>(stream);
  const dim3 grid((unsigned)((groups + 255) / 256));
  const bool vec = N % 8 == 0 && aligned16(out) && aligned16(gu);
#define GATE_MUL(ACT)                                                                                                                  \
  DISPATCH_T(dtype, if (vec) hipLaunchKernelGGL((gate_mul_kernel<T, ACT, true>), grid, dim3(256), 0, s, mp<T>(out), cp<T>(gu), (uint32_t)groups, N); \
             else hipLaunchKernelGGL((gate_mul_kernel<T, ACT, false>), grid, dim3(256), 0, s, mp<T>(out), cp<T>(gu), (uint32_t)groups, N);)
  if (act == MSGL_MIX_GATE_MUL_SILU) {
    GATE_MUL(MSGL_MIX_GATE_MUL_SILU)
  } else {
    GATE_MUL(MSGL_MIX_GATE_MUL_GELU_TANH)
  }
#undef GATE_MUL
  MIX_LAUNCHED("gate_mul");
  return MSGL_MIX_OK;
}

}  // extern "C"
