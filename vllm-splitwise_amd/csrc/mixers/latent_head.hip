// Attention over a low-rank latent whose queries come from a latent of their own, around the attention kernel:
//   * latent_down: one projection row holds [query latent | key latent | shared key part]; the query latent leaves
//     normed for its up-projection, the key latent normed and the key part rotated go into the paged cache;
//   * head_project: a product per head, out[t, h] = B[h] a[t, h], with what follows it fused in: next to it the
//     rotation of the head's other query coordinates (queries into the latent's space), or a sigmoid gate on the
//     result (the attention's output out of the latent's space, laid straight into a row of the next GEMM's input).
// Norms, angles, rotations, gates and sums are fp32; activations are read and written in the model's dtype.
#include "tile_gemm.cuh"

namespace swm {

// Rotation of `rot` coordinates: pair i is (i, i + rot / 2), or the neighbours (2i, 2i + 1); it turns by position *
// inv_freq[i] and grows by `amplitude`.
struct RotationParams {
  const int64_t* positions;
  const float* inv_freq;
  int rot, pair_halves;
  float amplitude;
};
__device__ __forceinline__ void rotation_of(const RotationParams& p, int64_t row, int i, int* u, int* v, float* c,
                                            float* s) {
  *u = p.pair_halves ? i : 2 * i;
  *v = p.pair_halves ? i + p.rot / 2 : 2 * i + 1;
  float sn, cs;
  sincosf((float)p.positions[row] * p.inv_freq[i], &sn, &cs);
  *c = cs * p.amplitude;
  *s = sn * p.amplitude;
}

constexpr int kLdThreads = 256;

// A wave per latent of a row: the even wave of a pair norms the query latent (or has nothing to do), the odd one norms the
// key latent, turns the key part and writes both into the cache.  V: neighbours per access (2: sizes, strides and bases
// are even); a latent of up to 512 numbers stays in registers between its sum and its scaling.
template <typename T, int V>
__device__ __forceinline__ void norm_latent(void* __restrict__ out, int64_t out_at, const void* __restrict__ in, int64_t at,
                                            int size, const float* __restrict__ weight, float eps) {
  using S = typename Conv<T>::store_t;
  struct alignas(V * sizeof(S)) Piece { S x[V]; };
  constexpr int PER = 512 / 64 / V;
  const int lane = threadIdx.x & 63;
  const S* src = static_cast<const S*>(in) + at;
  S* dst = static_cast<S*>(out) + out_at;
  auto get = [&](int c) { return *reinterpret_cast<const Piece*>(src + c); };
  Piece held[PER];
  float ss = 0.0f;
  auto add = [&](const Piece& p) {
#pragma unroll
    for (int e = 0; e < V; ++e) {
      const float x = Conv<T>::to_float(p.x[e]);
      ss += x * x;
    }
  };
#pragma unroll
  for (int j = 0; j < PER; ++j) {
    const int c = (lane + 64 * j) * V;
    if (c < size) {
      held[j] = get(c);
      add(held[j]);
    }
  }
  for (int c = (lane + 64 * PER) * V; c < size; c += 64 * V) add(get(c));
  const float f = 1.0f / sqrtf(sw::wave_sum(ss) / (float)size + eps);
  auto put = [&](int c, const Piece& p) {
    Piece o;
#pragma unroll
    for (int e = 0; e < V; ++e) o.x[e] = Conv<T>::from_float(Conv<T>::to_float(p.x[e]) * f * weight[c + e]);
    *reinterpret_cast<Piece*>(dst + c) = o;
  };
#pragma unroll
  for (int j = 0; j < PER; ++j) {
    const int c = (lane + 64 * j) * V;
    if (c < size) put(c, held[j]);
  }
  for (int c = (lane + 64 * PER) * V; c < size; c += 64 * V) put(c, get(c));
}

template <typename T, int V>
__global__ __launch_bounds__(kLdThreads) void latent_down_kernel(
    void* __restrict__ q_out, const void* __restrict__ q_down, int q_rank, const float* __restrict__ q_weight,
    const void* __restrict__ kv_down, int rank, const float* __restrict__ kv_weight, int64_t in_stride, float eps,
    RotationParams turn, void* __restrict__ cache, const int64_t* __restrict__ slot_mapping, int64_t rows) {
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int64_t t = (int64_t)blockIdx.x * (kLdThreads / 128) + (wave >> 1), in = t * in_stride;
  if (t >= rows) return;                                     // no barrier below
  if ((wave & 1) == 0) {
    if (q_rank > 0) norm_latent<T, V>(q_out, t * (int64_t)q_rank, q_down, in, q_rank, q_weight, eps);
    return;
  }
  const int64_t slot = slot_mapping[t];
  if (slot < 0) return;
  const int64_t dst = slot * (int64_t)(rank + turn.rot);
  for (int i = lane; i < turn.rot / 2; i += 64) {
    int u, v;
    float c, s;
    rotation_of(turn, t, i, &u, &v, &c, &s);
    const float a = ld<T>(kv_down, in + rank + u), b = ld<T>(kv_down, in + rank + v);
    st<T>(cache, dst + rank + u, a * c - b * s);
    st<T>(cache, dst + rank + v, b * c + a * s);
  }
  norm_latent<T, V>(cache, dst, kv_down, in, rank, kv_weight, eps);
}

// What a head_project launch reads and writes besides the tile loop's operands.
struct HeadProjectParams {
  int64_t rows, a_row, a_head, out_row, out_head, rot_row, rot_head, gate_row;
  int N, K;                    // B[h] is [N, K]
  int gate_per_head;           // gate column: head (per_head) or head * N + n
  int n_tiles;                 // workgroups with blockIdx.y >= n_tiles rotate
};

template <typename OUT, typename T>
__device__ __forceinline__ void head_store(void* out, const void* gate, const HeadProjectParams& p, int64_t t, int h,
                                           int n, float v) {
  if (gate != nullptr) v *= sigmoidf_(ld<T>(gate, t * p.gate_row + (p.gate_per_head ? h : h * p.N + n)));
  st<OUT>(out, t * p.out_row + h * p.out_head + n, v);
}

// coordinates N .. N + rot - 1 of out[t, h]: the rotated part of the query
template <typename OUT, typename T>
__device__ __forceinline__ void head_rotate(void* out, const void* q_rot, const HeadProjectParams& p,
                                            const RotationParams& turn, int64_t t0, int rows, int h) {
  const int pairs = turn.rot / 2;
  for (int e = threadIdx.x; e < rows * pairs; e += kTileThreads) {
    const int64_t t = t0 + e / pairs;
    int u, v;
    float c, s;
    rotation_of(turn, t, e % pairs, &u, &v, &c, &s);
    const int64_t src = t * p.rot_row + h * p.rot_head, dst = t * p.out_row + h * p.out_head + p.N;
    const float a = ld<T>(q_rot, src + u), b = ld<T>(q_rot, src + v);
    st<OUT>(out, dst + u, a * c - b * s);
    st<OUT>(out, dst + v, b * c + a * s);
  }
}

template <typename OUT>
__global__ __launch_bounds__(kTileThreads) void head_project_kernel(
    void* __restrict__ out, const float* __restrict__ a, const float* __restrict__ b, const float* __restrict__ q_rot,
    const float* __restrict__ gate, HeadProjectParams p, RotationParams turn) {
  __shared__ float As[TM][TK + 1];
  __shared__ float Bs[TN][TK + 1];
  const int64_t t0 = (int64_t)blockIdx.x * TM;
  const int rows = (int)min((int64_t)TM, p.rows - t0), h = blockIdx.z;
  if ((int)blockIdx.y >= p.n_tiles) {
    head_rotate<OUT, float>(out, q_rot, p, turn, t0, rows, h);
    return;
  }
  const int n0 = blockIdx.y * TN;
  float acc[2][4];
  tile_gemm<float>(acc, a, [&](int r) { return (t0 + r) * p.a_row + h * p.a_head; }, rows, b, (int64_t)h * p.N * p.K, n0,
                   p.N, p.K, As, Bs);
  const int ty = threadIdx.x >> 4, tx = threadIdx.x & 15;
#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int r = 2 * ty + i, n = n0 + tx + 16 * j;
      if (r < rows && n < p.N) head_store<OUT, float>(out, gate, p, t0 + r, h, n, acc[i][j]);
    }
}

template <typename OUT, bool VEC>
__global__ __launch_bounds__(kTileThreads) void head_project_mfma_kernel(
    void* __restrict__ out, const uint16_t* __restrict__ a, const uint16_t* __restrict__ b,
    const uint16_t* __restrict__ q_rot, const uint16_t* __restrict__ gate, HeadProjectParams p, RotationParams turn) {
  __shared__ __attribute__((aligned(16))) uint16_t As[MM][MK + MPAD];
  __shared__ __attribute__((aligned(16))) uint16_t Bs[MN][MK + MPAD];
  const int64_t t0 = (int64_t)blockIdx.x * MM;
  const int rows = (int)min((int64_t)MM, p.rows - t0), h = blockIdx.z;
  if ((int)blockIdx.y >= p.n_tiles) {
    head_rotate<OUT, bf16_t>(out, q_rot, p, turn, t0, rows, h);
    return;
  }
  const int n0 = blockIdx.y * MN;
  f32x16 acc;
  tile_gemm_mfma<VEC>(acc, a, [&](int r) { return (t0 + r) * p.a_row + h * p.a_head; }, rows, b, (int64_t)h * p.N * p.K,
                      n0, p.N, p.K, As, Bs);
  for_each_acc(acc, [&](int r, int c, float v) {
    if (r < rows && n0 + c < p.N) head_store<OUT, bf16_t>(out, gate, p, t0 + r, h, n0 + c, v);
  });
}

}  // namespace swm

extern "C" {

int swm_latent_down(void* q_out, const void* q_down, int q_rank, const float* q_weight, const void* kv_down, int rank,
                    const float* kv_weight, int64_t in_stride, float eps, const int64_t* positions,
                    const float* inv_freq, int rot, int pair_halves, float amplitude, void* cache,
                    const int64_t* slot_mapping, int64_t rows, int act_dtype, void* stream) {
  using namespace swm;
  if (rows == 0) return SW_OK;
  SW_CHECK_ARG(act_ok(act_dtype), "latent_down: unsupported dtype %d", act_dtype);
  SW_CHECK_ARG(rank > 0 && q_rank >= 0 && rot >= 0 && rot % 2 == 0 && rows < (1ll << 31),
               "latent_down: latents of %d and %d, %d rotated coordinates (an even number)", q_rank, rank, rot);
  SW_CHECK_ARG(kv_down != nullptr && kv_weight != nullptr && cache != nullptr && slot_mapping != nullptr &&
                   (q_rank == 0 || (q_down != nullptr && q_weight != nullptr && q_out != nullptr)) &&
                   (rot == 0 || (positions != nullptr && inv_freq != nullptr)),
               "latent_down: a part is missing");
  const RotationParams turn{positions, inv_freq, rot, pair_halves, amplitude};
  const uintptr_t piece = act_dtype == SW_F32 ? 8 : 4;
  auto even = [&](const void* p) { return reinterpret_cast<uintptr_t>(p) % piece == 0; };
  const bool pairs = q_rank % 2 == 0 && rank % 2 == 0 && in_stride % 2 == 0 && even(q_out) && even(q_down) &&
                     even(kv_down) && even(cache);
  const int per = kLdThreads / 128;
  const dim3 grid((unsigned)((rows + per - 1) / per));
  hipStream_t s = static_cast<hipStream_t>(stream);
  if (pairs) {
    SWM_DISPATCH_ACT(act_dtype, hipLaunchKernelGGL((latent_down_kernel<T, 2>), grid, dim3(kLdThreads), 0, s, q_out, q_down,
                                                   q_rank, q_weight, kv_down, rank, kv_weight, in_stride, eps, turn, cache,
                                                   slot_mapping, rows););
  } else {
    SWM_DISPATCH_ACT(act_dtype, hipLaunchKernelGGL((latent_down_kernel<T, 1>), grid, dim3(kLdThreads), 0, s, q_out, q_down,
                                                   q_rank, q_weight, kv_down, rank, kv_weight, in_stride, eps, turn, cache,
                                                   slot_mapping, rows););
  }
  SW_CHECK_LAUNCH();
  return SW_OK;
}

int swm_head_project(void* out, int out_dtype, int64_t out_row, int64_t out_head, const void* a, int64_t a_row,
                     int64_t a_head, const void* b, int N, int K, const void* q_rot, int64_t rot_row, int64_t rot_head,
                     const int64_t* positions, const float* inv_freq, int rot, int pair_halves, float amplitude,
                     const void* gate, int64_t gate_row, int gate_per_head, int64_t rows, int heads, int act_dtype,
                     void* stream) {
  using namespace swm;
  if (rows == 0) return SW_OK;
  SW_CHECK_ARG(act_ok(act_dtype) && (out_dtype == act_dtype || out_dtype == SW_F32),
               "head_project: unsupported dtypes %d -> %d", act_dtype, out_dtype);
  SW_CHECK_ARG(heads > 0 && heads <= 65535 && N > 0 && K > 0 && rot >= 0 && rot % 2 == 0 && rows < (1ll << 31),
               "head_project: %d heads of [%d, %d], %d rotated coordinates (an even number)", heads, N, K, rot);
  SW_CHECK_ARG(rot == 0 || (q_rot != nullptr && positions != nullptr && inv_freq != nullptr),
               "head_project: a rotated part needs its coordinates, positions and frequencies");
  const RotationParams turn{positions, inv_freq, rot, pair_halves, amplitude};
  const bool mfma = act_dtype == SW_BF16;
  const int tm = mfma ? MM : TM, n_tiles = (N + (mfma ? MN : TN) - 1) / (mfma ? MN : TN);
  const HeadProjectParams p{rows, a_row, a_head, out_row, out_head, rot_row, rot_head, gate_row, N, K, gate_per_head, n_tiles};
  const dim3 grid((unsigned)((rows + tm - 1) / tm), (unsigned)(n_tiles + (rot > 0 ? 1 : 0)), (unsigned)heads);
  hipStream_t s = static_cast<hipStream_t>(stream);
  if (!mfma) {
    hipLaunchKernelGGL(head_project_kernel<float>, grid, dim3(kTileThreads), 0, s, out, static_cast<const float*>(a),
                       static_cast<const float*>(b), static_cast<const float*>(q_rot), static_cast<const float*>(gate), p,
                       turn);
    SW_CHECK_LAUNCH();
    return SW_OK;
  }
  const bool vec = K % 8 == 0 && a_row % 8 == 0 && a_head % 8 == 0 && reinterpret_cast<uintptr_t>(a) % 16 == 0 &&
                   reinterpret_cast<uintptr_t>(b) % 16 == 0;
#define SWM_HEAD_CASE(OUT, VEC)                                                                                        \
  hipLaunchKernelGGL((head_project_mfma_kernel<OUT, VEC>), grid, dim3(kTileThreads), 0, s, out,                        \
                     static_cast<const uint16_t*>(a), static_cast<const uint16_t*>(b),                                 \
                     static_cast<const uint16_t*>(q_rot), static_cast<const uint16_t*>(gate), p, turn)
  if (out_dtype == SW_F32) {
    if (vec) SWM_HEAD_CASE(float, true);
    else SWM_HEAD_CASE(float, false);
  } else {
    if (vec) SWM_HEAD_CASE(bf16_t, true);
    else SWM_HEAD_CASE(bf16_t, false);
  }
#undef SWM_HEAD_CASE
  SW_CHECK_LAUNCH();
  return SW_OK;
}

}  // extern "C"
