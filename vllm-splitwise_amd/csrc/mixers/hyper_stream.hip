// A residual made of S parallel fp32 streams (hyper-connections): a sublayer reads one weighted sum of the streams and
// its output is written back to all of them while the streams are mixed with one another.
//   hyper_step: what lies between two sublayers, in one pass over the streams:
//         y     = a + b + c          or          blend * (N(a; wa) + N(b; wb))
//         x_j  <- sum_i mix[i, j] x_i + writes[j] * y            (all j from the old streams)
//         out   = N(sum_j reads[j] x_j; weight)                  (what the next sublayer reads)
//     with N(u; w) = u / sqrt(mean(u^2) + eps) * w.  At the start of a model all streams are equal to the embedding row:
//     the first launches take the old streams straight from the embedding table, so the S copies are never written.
//   gated_act: the activation between the two products of a gated feed-forward, act(gate) * up.
// All arithmetic is fp32; sublayer outputs and what a sublayer reads are in the model's dtype.
#include "mixers_common.cuh"

namespace swm {

constexpr int kMaxStreams = 8;
constexpr int kHyperMaxThreads = 1024;

struct HyperArgs {
  float* streams;              // [rows, S, width]
  const int64_t* ids;          // not NULL: every old stream of a row is table[ids[row]]
  const void* table;
  int64_t vocab;
  const float* mix;            // [S, S] (from, to); NULL: the streams stay as they are and are not written
  const float* writes;         // [S]
  const void *a, *b;           // sublayer outputs (activation type), row strides
  int64_t a_stride, b_stride;
  const float* c;              // a further addend, fp32 [rows, width]
  const float *wa, *wb;        // not NULL: y = blend * (N(a; wa) + N(b; wb))
  float blend;
  const float* reads;          // [S]
  const float* weight;         // [width]
  float eps;
  void* out;                   // [rows, width]
  int width;
};

// One workgroup per row; a thread owns P pieces of V neighbouring channels and keeps all S streams of them, and the sum
// that the next sublayer reads, in registers.
template <typename T, int S, int V, int P>
__global__ __launch_bounds__(kHyperMaxThreads) void hyper_step_kernel(HyperArgs g) {
  __shared__ float red[16];
  const int64_t t = blockIdx.x;
  const int width = g.width;
  float* xrow = g.streams + t * S * (int64_t)width;
  int at[P];                                                 // first channel of every piece; clamped where there is none
  bool live[P];
#pragma unroll
  for (int p = 0; p < P; ++p) {
    const int c = ((int)threadIdx.x + p * (int)blockDim.x) * V;
    live[p] = c < width;
    at[p] = live[p] ? c : 0;
  }
  // ---- the old streams
  float x[P][S][V];
  if (g.ids != nullptr) {
    const int64_t id = g.ids[t];
    const bool known = id >= 0 && id < g.vocab;              // an id beyond the table reads nothing and shows as NaN
    const int64_t src = known ? id * width : 0;
#pragma unroll
    for (int p = 0; p < P; ++p) {
      float e[V];
      ld_vec<T, V>(e, g.table, src + at[p]);
#pragma unroll
      for (int s = 0; s < S; ++s)
#pragma unroll
        for (int j = 0; j < V; ++j) x[p][s][j] = known ? e[j] : __builtin_nanf("");
    }
  } else {
#pragma unroll
    for (int p = 0; p < P; ++p)
#pragma unroll
      for (int s = 0; s < S; ++s) ld_vec<float, V>(x[p][s], xrow, (int64_t)s * width + at[p]);
  }
  // ---- the sublayer's output, mixed in
  if (g.mix != nullptr) {
    float y[P][V];
    if (g.wa != nullptr) {
      float ya[P][V], yb[P][V], sa = 0.0f, sb = 0.0f;
#pragma unroll
      for (int p = 0; p < P; ++p) {
        ld_vec<T, V>(ya[p], g.a, t * g.a_stride + at[p]);
        ld_vec<T, V>(yb[p], g.b, t * g.b_stride + at[p]);
      }
#pragma unroll
      for (int p = 0; p < P; ++p)
#pragma unroll
        for (int j = 0; j < V; ++j) {
          sa += live[p] ? ya[p][j] * ya[p][j] : 0.0f;
          sb += live[p] ? yb[p][j] * yb[p][j] : 0.0f;
        }
      sa = block_sum(sa, red);
      sb = block_sum(sb, red);
      const float fa = g.blend / sqrtf(sa / (float)width + g.eps), fb = g.blend / sqrtf(sb / (float)width + g.eps);
#pragma unroll
      for (int p = 0; p < P; ++p) {
        float wa[V], wb[V];
        ld_vec<float, V>(wa, g.wa, at[p]);
        ld_vec<float, V>(wb, g.wb, at[p]);
#pragma unroll
        for (int j = 0; j < V; ++j) y[p][j] = ya[p][j] * fa * wa[j] + yb[p][j] * fb * wb[j];
      }
    } else {
#pragma unroll
      for (int p = 0; p < P; ++p) {
#pragma unroll
        for (int j = 0; j < V; ++j) y[p][j] = 0.0f;
        float v[V];
        if (g.a != nullptr) {
          ld_vec<T, V>(v, g.a, t * g.a_stride + at[p]);
#pragma unroll
          for (int j = 0; j < V; ++j) y[p][j] += v[j];
        }
        if (g.b != nullptr) {
          ld_vec<T, V>(v, g.b, t * g.b_stride + at[p]);
#pragma unroll
          for (int j = 0; j < V; ++j) y[p][j] += v[j];
        }
        if (g.c != nullptr) {
          ld_vec<float, V>(v, g.c, t * (int64_t)width + at[p]);
#pragma unroll
          for (int j = 0; j < V; ++j) y[p][j] += v[j];
        }
      }
    }
#pragma unroll
    for (int p = 0; p < P; ++p) {
      float n[S][V];
#pragma unroll
      for (int to = 0; to < S; ++to) {
        const float w = g.writes[to];
#pragma unroll
        for (int j = 0; j < V; ++j) n[to][j] = w * y[p][j];
#pragma unroll
        for (int from = 0; from < S; ++from) {
          const float m = g.mix[from * S + to];
#pragma unroll
          for (int j = 0; j < V; ++j) n[to][j] += m * x[p][from][j];
        }
      }
#pragma unroll
      for (int s = 0; s < S; ++s) {
#pragma unroll
        for (int j = 0; j < V; ++j) x[p][s][j] = n[s][j];
        if (live[p]) st_vec<float, V>(xrow, (int64_t)s * width + at[p], n[s]);
      }
    }
  }
  if (g.out == nullptr) return;                              // the whole grid
  // ---- what the next sublayer reads
  float u[P][V], ss = 0.0f;
#pragma unroll
  for (int p = 0; p < P; ++p)
#pragma unroll
    for (int j = 0; j < V; ++j) {
      float v = 0.0f;
#pragma unroll
      for (int s = 0; s < S; ++s) v += g.reads[s] * x[p][s][j];
      u[p][j] = v;
      ss += live[p] ? v * v : 0.0f;
    }
  ss = block_sum(ss, red);
  const float f = 1.0f / sqrtf(ss / (float)width + g.eps);
#pragma unroll
  for (int p = 0; p < P; ++p) {
    float w[V];
    ld_vec<float, V>(w, g.weight, at[p]);
#pragma unroll
    for (int j = 0; j < V; ++j) u[p][j] *= f * w[j];
    if (live[p]) st_vec<T, V>(g.out, t * (int64_t)width + at[p], u[p]);
  }
}

template <typename T, int S>
int launch_hyper_step(const HyperArgs& g, int64_t rows, bool vec, hipStream_t stream) {
  const int pieces = vec ? g.width / 4 : g.width;
  // two pieces of a row per thread where the row is long enough, more only beyond 1024 threads
  auto threads_for = [&](int per) { return std::max(64, (pieces + per * 64 - 1) / (per * 64) * 64); };
  const dim3 grid((unsigned)rows);
#define SWM_HYPER_LAUNCH(VV, PP)                                                                                     \
  do {                                                                                                               \
    hipLaunchKernelGGL((hyper_step_kernel<T, S, VV, PP>), grid, dim3((unsigned)threads_for(PP)), 0, stream, g);      \
    SW_CHECK_LAUNCH();                                                                                               \
    return SW_OK;                                                                                                    \
  } while (0)
  if (vec) {
    if (pieces <= 128) SWM_HYPER_LAUNCH(4, 1);
    if (threads_for(2) <= kHyperMaxThreads) SWM_HYPER_LAUNCH(4, 2);
    if (threads_for(4) <= kHyperMaxThreads) SWM_HYPER_LAUNCH(4, 4);
  } else if (threads_for(8) <= kHyperMaxThreads) {
    SWM_HYPER_LAUNCH(1, 8);
  }
#undef SWM_HYPER_LAUNCH
  sw::set_error("hyper_step: a row of %d channels is too wide (at most %d, or %d off multiples of 4)", g.width,
                kHyperMaxThreads * 16, kHyperMaxThreads * 8);
  return SW_ERR_INVALID;
}

// act(gate) * up of a row [gate | up], both activations of the form z * sigmoid(r(z)):
// silu: r = z; the tanh form of gelu: 0.5 z (1 + tanh(v)) = z * sigmoid(2 v), v = sqrt(2 / pi) (z + 0.044715 z^3)
__device__ __forceinline__ float gate_act(float z, int act) {
  const float r = act == SWM_GATE_GELU_TANH ? 1.5957691216057308f * (z + 0.044715f * z * z * z) : z;
  return z * __builtin_amdgcn_rcpf(1.0f + fast_expf_(-r));
}

template <typename T, int V>
__global__ __launch_bounds__(256) void gated_act_kernel(void* __restrict__ out, int64_t out_stride,
                                                        const void* __restrict__ in, int64_t in_stride, int ff, int act) {
  const int64_t t = blockIdx.x;
  for (int c = ((int)blockIdx.y * 256 + (int)threadIdx.x) * V; c < ff; c += (int)gridDim.y * 256 * V) {
    float z[V], u[V];
    ld_vec<T, V>(z, in, t * in_stride + c);
    ld_vec<T, V>(u, in, t * in_stride + ff + c);
#pragma unroll
    for (int j = 0; j < V; ++j) z[j] = gate_act(z[j], act) * u[j];
    st_vec<T, V>(out, t * out_stride + c, z);
  }
}

}  // namespace swm

extern "C" {

int swm_hyper_step(float* streams, int num_streams, const int64_t* ids, const void* table, int64_t vocab,
                   const float* mix, const float* writes, const void* a, int64_t a_stride, const void* b,
                   int64_t b_stride, const float* c, const float* a_norm, const float* b_norm, float blend,
                   const float* reads, const float* weight, float eps, void* out, int64_t rows, int width, int act_dtype,
                   void* stream) {
  using namespace swm;
  if (rows == 0) return SW_OK;
  SW_CHECK_ARG(act_ok(act_dtype), "hyper_step: unsupported dtype %d", act_dtype);
  SW_CHECK_ARG(num_streams >= 1 && num_streams <= kMaxStreams, "hyper_step: %d streams (1..%d supported)", num_streams,
               kMaxStreams);
  SW_CHECK_ARG(width > 0 && rows < (1ll << 31), "hyper_step: bad shape");
  SW_CHECK_ARG((ids == nullptr) == (table == nullptr) && (ids == nullptr || vocab > 0), "hyper_step: ids go with a table");
  SW_CHECK_ARG((mix == nullptr) == (writes == nullptr), "hyper_step: the streams' mix goes with their writes");
  SW_CHECK_ARG((a_norm == nullptr) == (b_norm == nullptr) && (a_norm == nullptr || (a != nullptr && b != nullptr && c == nullptr)),
               "hyper_step: normed outputs come in twos");
  SW_CHECK_ARG(out == nullptr || (reads != nullptr && weight != nullptr), "hyper_step: an output needs reads and a norm");
  SW_CHECK_ARG(streams != nullptr || (mix == nullptr && ids != nullptr), "hyper_step: no streams");
  const HyperArgs g{streams, ids, table, vocab, mix, writes, a, b, a_stride, b_stride, c, a_norm, b_norm, blend, reads, weight,
                    eps, out, width};
  const uintptr_t piece = act_dtype == SW_F32 ? 16 : 8;
  auto on = [](const void* p, uintptr_t n) { return reinterpret_cast<uintptr_t>(p) % n == 0; };
  const bool vec = width % 4 == 0 && a_stride % 4 == 0 && b_stride % 4 == 0 && on(a, piece) && on(b, piece) && on(table, piece) &&
                   on(out, piece) && on(streams, 16) && on(c, 16) && on(a_norm, 16) && on(b_norm, 16) && on(weight, 16);
  hipStream_t s = static_cast<hipStream_t>(stream);
#define SWM_HYPER_CASE(N) \
  case N: SWM_DISPATCH_ACT(act_dtype, return (launch_hyper_step<T, N>(g, rows, vec, s));); break;
  switch (num_streams) {
    SWM_HYPER_CASE(1)
    SWM_HYPER_CASE(2)
    SWM_HYPER_CASE(3)
    SWM_HYPER_CASE(4)
    SWM_HYPER_CASE(5)
    SWM_HYPER_CASE(6)
    SWM_HYPER_CASE(7)
    SWM_HYPER_CASE(8)
  }
#undef SWM_HYPER_CASE
  return SW_OK;
}

int swm_gated_act(void* out, int64_t out_stride, const void* in, int64_t in_stride, int64_t rows, int ff, int activation,
                  int act_dtype, void* stream) {
  using namespace swm;
  if (rows == 0) return SW_OK;
  SW_CHECK_ARG(act_ok(act_dtype), "gated_act: unsupported dtype %d", act_dtype);
  SW_CHECK_ARG(activation == SWM_GATE_SILU || activation == SWM_GATE_GELU_TANH, "gated_act: unknown activation %d", activation);
  SW_CHECK_ARG(ff > 0 && out_stride >= ff && in_stride >= 2 * (int64_t)ff && rows < (1ll << 31), "gated_act: bad shape");
  hipStream_t s = static_cast<hipStream_t>(stream);
  const int v = act_dtype == SW_F32 ? 4 : 8;
  if (ff % v == 0 && in_stride % v == 0 && out_stride % v == 0 && reinterpret_cast<uintptr_t>(in) % 16 == 0 &&
      reinterpret_cast<uintptr_t>(out) % 16 == 0) {
    const dim3 grid((unsigned)rows, (unsigned)std::min(8, (ff / v + 255) / 256));
    if (act_dtype == SW_F32)
      hipLaunchKernelGGL((gated_act_kernel<float, 4>), grid, dim3(256), 0, s, out, out_stride, in, in_stride, ff, activation);
    else
      hipLaunchKernelGGL((gated_act_kernel<bf16_t, 8>), grid, dim3(256), 0, s, out, out_stride, in, in_stride, ff, activation);
  } else {
    const dim3 grid((unsigned)rows, (unsigned)std::min(8, (ff + 255) / 256));
    SWM_DISPATCH_ACT(act_dtype, hipLaunchKernelGGL((gated_act_kernel<T, 1>), grid, dim3(256), 0, s, out, out_stride, in,
                                                   in_stride, ff, activation););
  }
  SW_CHECK_LAUNCH();
  return SW_OK;
}

}  // extern "C"
