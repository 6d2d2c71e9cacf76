// From a layer's input projections to what its token mixers read, one launch for a layer with one mixer or two side by
// side on the same projection output:
//   * softmax attention: queries and keys optionally take ONE RMS norm over the whole projection (all heads together),
//     then the rotary embedding; queries leave in fp32, keys and values go to the paged cache;
//   * linear attention: queries and keys take the rotary embedding and leave in fp32, the keys times a factor.
// Rotation: coordinate i < rot / 2 of a head turns with coordinate i + rot / 2 by float(position) * inv_freq[i], the rest of
// the head passes.  A row's sines and cosines are worked out once, in LDS, for all heads of queries and keys.
// All arithmetic is fp32.
#include "mixers_common.cuh"

namespace swm {

constexpr int kRopeThreads = 256;
constexpr int kMaxPairs = 256;          // rotated pairs of a head

struct RopeSide {
  const void *q, *k, *v;       // column ranges of the projection output (NULL q: no such mixer)
  const float *q_norm, *k_norm;
  const float* inv_freq;
  int rot, heads, kv_heads, dim, vdim;
  float k_scale;
  float* q_out;                // [rows, heads * dim]
  void* k_out;                 // attention: the key cache; linear: fp32 [rows, heads * dim]
  void* v_out;                 // attention: the value cache
};

// V: neighbours per access (1: any sizes and strides).  The heads at src[off ..] turned: dst[dst_off ..] = scale * rotate(x * fac * norm)
template <typename T, typename TO, int V>
__device__ __forceinline__ void turn_heads(void* __restrict__ dst, int64_t dst_off, const void* __restrict__ src, int64_t off,
                                           int heads, int dim, int half, float fac, const float* __restrict__ norm,
                                           const float* cs, const float* sn, float scale) {
  const int units = (dim - half) / V;                        // per head: half / V of pairs, the rest pass
  for (int e = threadIdx.x; e < heads * units; e += kRopeThreads) {
    const int h = e / units, i = (e % units) * V, base = h * dim;
    float a[V];
    if (i < half) {
      float b[V];
      ld_vec<T, V>(a, src, off + base + i);
      ld_vec<T, V>(b, src, off + base + i + half);
      if (norm != nullptr) {
#pragma unroll
        for (int j = 0; j < V; ++j) {
          a[j] *= fac * norm[base + i + j];
          b[j] *= fac * norm[base + i + half + j];
        }
      }
#pragma unroll
      for (int j = 0; j < V; ++j) {
        const float c = cs[i + j], s = sn[i + j], u = a[j], w = b[j];
        a[j] = (u * c - w * s) * scale;
        b[j] = (w * c + u * s) * scale;
      }
      st_vec<TO, V>(dst, dst_off + base + i, a);
      st_vec<TO, V>(dst, dst_off + base + i + half, b);
    } else {
      ld_vec<T, V>(a, src, off + base + i + half);
#pragma unroll
      for (int j = 0; j < V; ++j) a[j] *= (norm != nullptr ? fac * norm[base + i + half + j] : 1.0f) * scale;
      st_vec<TO, V>(dst, dst_off + base + i + half, a);
    }
  }
}

template <typename T>
__device__ __forceinline__ float square_sum(const void* __restrict__ src, int64_t off, int n, float* red) {
  float ss = 0.0f;
  for (int i = threadIdx.x; i < n; i += kRopeThreads) {
    const float x = ld<T>(src, off + i);
    ss += x * x;
  }
  return block_sum(ss, red);
}

// grid (rows, 2): blockIdx.y 0: the attention side, 1: the linear side
template <typename T, int VA, int VL>
__global__ __launch_bounds__(kRopeThreads) void rope_operands_kernel(RopeSide att, RopeSide lin, int64_t in_stride,
                                                                     const int64_t* __restrict__ positions,
                                                                     const int64_t* __restrict__ slot_mapping,
                                                                     float norm_eps) {
  __shared__ float cs[kMaxPairs], sn[kMaxPairs], red[16];
  const int64_t t = blockIdx.x, row = t * in_stride;
  const bool linear = att.q == nullptr || blockIdx.y == 1;
  const RopeSide& s = linear ? lin : att;
  const float pos = (float)positions[t];
  const int half = s.rot / 2;
  for (int i = threadIdx.x; i < half; i += kRopeThreads) sincosf(pos * s.inv_freq[i], &sn[i], &cs[i]);
  const int qn = s.heads * s.dim, kn = s.kv_heads * s.dim;
  if (linear) {
    __syncthreads();
    turn_heads<T, float, VL>(s.q_out, t * qn, s.q, row, s.heads, s.dim, half, 1.0f, nullptr, cs, sn, 1.0f);
    turn_heads<T, float, VL>(s.k_out, t * kn, s.k, row, s.kv_heads, s.dim, half, 1.0f, nullptr, cs, sn, s.k_scale);
    return;
  }
  float fq = 1.0f, fk = 1.0f;
  if (s.q_norm != nullptr) {
    fq = 1.0f / sqrtf(square_sum<T>(s.q, row, qn, red) / (float)qn + norm_eps);
    fk = 1.0f / sqrtf(square_sum<T>(s.k, row, kn, red) / (float)kn + norm_eps);
  }
  __syncthreads();
  turn_heads<T, float, VA>(s.q_out, t * qn, s.q, row, s.heads, s.dim, half, fq, s.q_norm, cs, sn, 1.0f);
  const int64_t slot = slot_mapping[t];
  if (slot < 0) return;
  turn_heads<T, T, VA>(s.k_out, slot * kn, s.k, row, s.kv_heads, s.dim, half, fk, s.k_norm, cs, sn, s.k_scale);
  const int vn = s.kv_heads * s.vdim;
  for (int i = threadIdx.x; i < vn; i += kRopeThreads) st<T>(s.v_out, slot * vn + i, ld<T>(s.v, row + i));
}

}  // namespace swm

extern "C" int swm_rope_operands(float* q_out, const void* q, const void* k, const void* v, const float* q_norm,
                                 const float* k_norm, float norm_eps, const float* inv_freq, int rot, int heads, int kv_heads,
                                 int dim, int vdim, void* key_cache, void* value_cache, const int64_t* slot_mapping,
                                 float* lin_q_out, float* lin_k_out, const void* lin_q, const void* lin_k,
                                 const float* lin_inv_freq, int lin_rot, int lin_heads, int lin_dim, float lin_k_scale,
                                 const int64_t* positions, int64_t in_stride, int64_t rows, int act_dtype, void* stream) {
  using namespace swm;
  if (rows == 0) return SW_OK;
  SW_CHECK_ARG(act_ok(act_dtype), "rope_operands: unsupported dtype %d", act_dtype);
  SW_CHECK_ARG((q != nullptr || lin_q != nullptr) && positions != nullptr && rows < (1ll << 31), "rope_operands: nothing to do");
  auto side_ok = [](int hd, int d, int r, const float* f) {
    return hd > 0 && d > 0 && r >= 0 && r % 2 == 0 && r <= d && r <= 2 * kMaxPairs && (r == 0 || f != nullptr);
  };
  if (q != nullptr) {
    SW_CHECK_ARG(side_ok(heads, dim, rot, inv_freq), "rope_operands: %d heads of %d, %d rotated", heads, dim, rot);
    SW_CHECK_ARG(k != nullptr && v != nullptr && q_out != nullptr && key_cache != nullptr && value_cache != nullptr &&
                     slot_mapping != nullptr && kv_heads > 0 && vdim > 0 && (q_norm == nullptr) == (k_norm == nullptr),
                 "rope_operands: a part of the attention side is missing");
  }
  if (lin_q != nullptr) {
    SW_CHECK_ARG(side_ok(lin_heads, lin_dim, lin_rot, lin_inv_freq), "rope_operands: %d heads of %d, %d rotated", lin_heads,
                 lin_dim, lin_rot);
    SW_CHECK_ARG(lin_k != nullptr && lin_q_out != nullptr && lin_k_out != nullptr, "rope_operands: a part of the linear side is missing");
  }
  const RopeSide att{q, k, v, q_norm, k_norm, inv_freq, rot, heads, kv_heads, dim, vdim, 1.0f, q_out, key_cache, value_cache};
  const RopeSide lin{lin_q, lin_k, nullptr, nullptr, nullptr, lin_inv_freq, lin_rot, lin_heads, lin_heads, lin_dim, 0,
                     lin_k_scale, lin_q_out, lin_k_out, nullptr};
  // pieces of 4 where every head's halves, its passing rest, the strides and the bases allow it
  const uintptr_t piece = act_dtype == SW_F32 ? 16 : 8;
  auto on = [](const void* p, uintptr_t n) { return reinterpret_cast<uintptr_t>(p) % n == 0; };
  const bool av = q == nullptr || (dim % 4 == 0 && rot % 8 == 0 && in_stride % 4 == 0 && on(q, piece) && on(k, piece) &&
                                   on(key_cache, piece) && on(q_out, 16));
  const bool lv = lin_q == nullptr || (lin_dim % 4 == 0 && lin_rot % 8 == 0 && in_stride % 4 == 0 && on(lin_q, piece) &&
                                       on(lin_k, piece) && on(lin_q_out, 16) && on(lin_k_out, 16));
  const dim3 grid((unsigned)rows, q != nullptr && lin_q != nullptr ? 2u : 1u);
  hipStream_t s = static_cast<hipStream_t>(stream);
#define SWM_ROPE_LAUNCH(A, L)                                                                                              \
  SWM_DISPATCH_ACT(act_dtype, hipLaunchKernelGGL((rope_operands_kernel<T, A, L>), grid, dim3(kRopeThreads), 0, s, att, lin, \
                                                 in_stride, positions, slot_mapping, norm_eps);)
  if (av && lv) SWM_ROPE_LAUNCH(4, 4);
  else if (av) SWM_ROPE_LAUNCH(4, 1);
  else if (lv) SWM_ROPE_LAUNCH(1, 4);
  else SWM_ROPE_LAUNCH(1, 1);
#undef SWM_ROPE_LAUNCH
  SW_CHECK_LAUNCH();
  return SW_OK;
}
