// The fp32 stream of a decoder that runs a block of its layers several times: where the stream begins and where a
// pass begins.
//   * embed_stream: the stream's first value, scale * embedding row, the row itself in the activation dtype (what a
//     pass's input projection multiplies: the scale is applied to the product) and the first norm, in one pass;
//   * stream_split: a layer's outputs are summed into the stream and the new stream leaves as a pair of bf16 numbers
//     [high | low], high + low = the fp32 value to 16 bits of mantissa, so that a bf16 product of it accumulated in fp32
//     does not round the stream to bf16.
#include "mixers_common.cuh"

namespace swm {

constexpr int kLsThreads = 256;

template <typename T>
__global__ __launch_bounds__(kLsThreads) void embed_stream_kernel(
    float* __restrict__ stream, void* __restrict__ rows_out, const int64_t* __restrict__ ids,
    const void* __restrict__ table, int64_t vocab, float scale, const float* __restrict__ weight, float offset, float eps,
    void* __restrict__ out, int width) {
  __shared__ float red[16];
  const int64_t t = blockIdx.x, id = ids[t];
  const bool known = id >= 0 && id < vocab;                  // an id beyond the table reads nothing and shows as NaN
  const int64_t src = known ? id * width : 0, dst = t * (int64_t)width;
  float ss = 0.0f;
  for (int i = threadIdx.x; i < width; i += kLsThreads) {
    const float e = known ? ld<T>(table, src + i) : __builtin_nanf("");
    const float v = e * scale;
    stream[dst + i] = v;
    if (rows_out != nullptr) st<T>(rows_out, dst + i, e);
    ss += v * v;
  }
  if (out == nullptr) return;
  ss = block_sum(ss, red);
  const float f = 1.0f / sqrtf(ss / (float)width + eps);
  for (int i = threadIdx.x; i < width; i += kLsThreads) st<T>(out, dst + i, stream[dst + i] * f * (offset + weight[i]));
}

// grid (rows, pieces of a row)
__global__ __launch_bounds__(kLsThreads) void stream_split_kernel(
    float* __restrict__ stream, const void* __restrict__ a, int64_t a_stride, const void* __restrict__ b, int64_t b_stride,
    const float* __restrict__ c, void* __restrict__ split, int width) {
  const int64_t t = blockIdx.x;
  for (int i = blockIdx.y * kLsThreads + threadIdx.x; i < width; i += gridDim.y * kLsThreads) {
    float v = stream[t * (int64_t)width + i];
    if (a != nullptr || b != nullptr || c != nullptr) {
      float add = 0.0f;
      if (a != nullptr) add += ld<bf16_t>(a, t * a_stride + i);
      if (b != nullptr) add += ld<bf16_t>(b, t * b_stride + i);
      if (c != nullptr) add += c[t * (int64_t)width + i];
      v += add;
      stream[t * (int64_t)width + i] = v;
    }
    const uint16_t high = sw::float_to_bf16_bits(v);
    static_cast<uint16_t*>(split)[t * 2 * (int64_t)width + i] = high;
    st<bf16_t>(split, t * 2 * (int64_t)width + width + i, v - sw::bf16_bits_to_float(high));
  }
}

}  // namespace swm

extern "C" {

int swm_embed_stream(float* stream_out, void* rows_out, const int64_t* ids, const void* table, int64_t vocab, float scale,
                     const float* weight, float offset, float eps, void* out, int64_t rows, int width, int act_dtype,
                     void* stream) {
  using namespace swm;
  if (rows == 0) return SW_OK;
  SW_CHECK_ARG(act_ok(act_dtype), "embed_stream: unsupported dtype %d", act_dtype);
  SW_CHECK_ARG(width > 0 && vocab > 0 && rows < (1ll << 31) && (out == nullptr || weight != nullptr),
               "embed_stream: bad shape, or a norm without its weight");
  SWM_DISPATCH_ACT(act_dtype, hipLaunchKernelGGL(embed_stream_kernel<T>, dim3((unsigned)rows), dim3(kLsThreads), 0,
                                                 static_cast<hipStream_t>(stream), stream_out, rows_out, ids, table, vocab,
                                                 scale, weight, offset, eps, out, width););
  SW_CHECK_LAUNCH();
  return SW_OK;
}

int swm_stream_split(float* stream_io, const void* a, int64_t a_stride, const void* b, int64_t b_stride, const float* c,
                     void* split, int64_t rows, int width, void* stream) {
  using namespace swm;
  if (rows == 0) return SW_OK;
  SW_CHECK_ARG(width > 0 && rows < (1ll << 31) && split != nullptr, "stream_split: bad shape");
  const dim3 grid((unsigned)rows, (unsigned)std::min(8, (width + 4 * kLsThreads - 1) / (4 * kLsThreads)));
  hipLaunchKernelGGL(stream_split_kernel, grid, dim3(kLsThreads), 0, static_cast<hipStream_t>(stream), stream_io, a,
                     a_stride, b, b_stride, c, split, width);
  SW_CHECK_LAUNCH();
  return SW_OK;
}

}  // extern "C"
