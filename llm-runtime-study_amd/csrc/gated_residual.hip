// The stream's update in layers that gate and normalise what a sublayer gives out, and the activation of their feed-forward.
//
//   gated_norm_add  per token: the sublayer's output y times the sigmoid of a gate row (z + bias), divided by its root mean square,
//                   times a weight per column, added into the float32 stream; and beside the new stream its RMS norm, the input
//                   of the sublayer that runs next;
//   xielu           act(z) = a z^2 + z / 2 for z > 0, b (exp(z) - 1 - z) + z / 2 otherwise, a and b two numbers of the layer.
#include "common.h"

namespace {

template <typename TZ, typename TN>
__global__ __launch_bounds__(256) void gated_norm_add_kernel(float* __restrict__ stream, const float* __restrict__ y, const TZ* __restrict__ z,
                                                             int z_stride, const float* __restrict__ z_bias, const float* __restrict__ weight,
                                                             float eps, int cols, const float* __restrict__ next_weight, float next_eps,
                                                             TN* __restrict__ normed) {
  __shared__ float scratch[16];
  const int64_t base = (int64_t)blockIdx.x * cols;
  const TZ* zrow = z ? z + (int64_t)blockIdx.x * z_stride : nullptr;
  auto gated = [&](int c) {
    const float v = y[base + c];
    return zrow ? v / (1.f + expf(-(to_float(zrow[c]) + (z_bias ? z_bias[c] : 0.f)))) : v;
  };
  float ss = 0.f;
  for (int c = threadIdx.x; c < cols; c += 256) {
    const float v = gated(c);
    ss = fmaf(v, v, ss);
  }
  ss = block_sum(ss, scratch);
  const float inv = 1.0f / sqrtf(ss / (float)cols + eps);
  float next = 0.f;
  for (int c = threadIdx.x; c < cols; c += 256) {
    const float v = stream[base + c] + gated(c) * inv * weight[c];
    stream[base + c] = v;
    next = fmaf(v, v, next);
  }
  if (!normed) return;
  next = block_sum(next, scratch);
  const float next_inv = 1.0f / sqrtf(next / (float)cols + next_eps);
  for (int c = threadIdx.x; c < cols; c += 256) normed[base + c] = from_float<TN>(stream[base + c] * next_inv * next_weight[c]);
}

// The same for rows of up to 8,192 values, a multiple of four: 16 bytes a load of the float32 rows (eight of a bfloat16 gate row),
// every load on its way before the first is used, the row in registers from the first sum to the last store.
template <typename TZ, typename TN, int THREADS>
__global__ __launch_bounds__(THREADS) void gated_norm_add_vec_kernel(float* __restrict__ stream, const float* __restrict__ y, const TZ* __restrict__ z,
                                                                     int z_stride, const float* __restrict__ z_bias,
                                                                     const float* __restrict__ weight, float eps, int cols,
                                                                     const float* __restrict__ next_weight, float next_eps, TN* __restrict__ normed) {
  constexpr int PER = 8192 / 4 / THREADS;
  typedef TZ z4 __attribute__((ext_vector_type(4)));
  __shared__ float scratch[16];
  const int64_t base = (int64_t)blockIdx.x * cols;
  const int quads = cols / 4;
  floatx4 vy[PER], vs[PER], vb[PER], vw[PER], vn[PER];
  z4 vz[PER];
#pragma unroll
  for (int n = 0; n < PER; ++n) {
    const int q = threadIdx.x + n * THREADS;
    if (q < quads) {
      vy[n] = *(const floatx4*)(y + base + 4 * q);
      if (z) {
        vz[n] = *(const z4*)(z + (int64_t)blockIdx.x * z_stride + 4 * q);
        vb[n] = z_bias ? *(const floatx4*)(z_bias + 4 * q) : floatx4{0.f, 0.f, 0.f, 0.f};
      }
      vs[n] = *(const floatx4*)(stream + base + 4 * q);
      vw[n] = *(const floatx4*)(weight + 4 * q);
      if (normed) vn[n] = *(const floatx4*)(next_weight + 4 * q);
    }
  }
  float ss = 0.f;
#pragma unroll
  for (int n = 0; n < PER; ++n) {
    if (threadIdx.x + n * THREADS < quads) {
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        if (z) vy[n][i] = vy[n][i] / (1.f + expf(-((float)vz[n][i] + vb[n][i])));
        ss = fmaf(vy[n][i], vy[n][i], ss);
      }
    }
  }
  ss = block_sum(ss, scratch);
  const float inv = 1.0f / sqrtf(ss / (float)cols + eps);
  float next = 0.f;
#pragma unroll
  for (int n = 0; n < PER; ++n) {
    const int q = threadIdx.x + n * THREADS;
    if (q < quads) {
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        vs[n][i] = vs[n][i] + vy[n][i] * inv * vw[n][i];
        next = fmaf(vs[n][i], vs[n][i], next);
      }
      *(floatx4*)(stream + base + 4 * q) = vs[n];
    }
  }
  if (!normed) return;
  next = block_sum(next, scratch);
  const float next_inv = 1.0f / sqrtf(next / (float)cols + next_eps);
#pragma unroll
  for (int n = 0; n < PER; ++n) {
    const int q = threadIdx.x + n * THREADS;
    if (q < quads) {
      typedef TN n4 __attribute__((ext_vector_type(4)));
      n4 packed;
#pragma unroll
      for (int i = 0; i < 4; ++i) packed[i] = from_float<TN>(vs[n][i] * next_inv * vn[n][i]);
      *(n4*)(normed + base + 4 * q) = packed;
    }
  }
}

__device__ __forceinline__ float xielu(float z, float a, float b) {
  return z > 0.f ? fmaf(a * z, z, 0.5f * z) : fmaf(b, expm1f(z) - z, 0.5f * z);
}

template <typename T>
__global__ __launch_bounds__(256) void xielu_kernel(T* __restrict__ out, int out_stride, const T* __restrict__ x, int x_stride, int64_t pieces,
                                                    int per_row, int cols, const float* __restrict__ numbers) {
  constexpr int RUN = 16 / sizeof(T);
  typedef T vec __attribute__((ext_vector_type(RUN)));
  const int64_t e = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (e >= pieces) return;
  const int64_t row = e / per_row;
  const int at = (int)(e % per_row) * RUN;
  const float a = numbers[0], b = numbers[1];
  const T* src = x + row * x_stride + at;
  T* dst = out + row * out_stride + at;
  if (at + RUN <= cols && ((uintptr_t)src | (uintptr_t)dst) % 16 == 0) {
    vec v = *(const vec*)src;
#pragma unroll
    for (int i = 0; i < RUN; ++i) v[i] = from_float<T>(xielu(to_float(v[i]), a, b));
    *(vec*)dst = v;
  } else {
    for (int i = 0; i < RUN && at + i < cols; ++i) dst[i] = from_float<T>(xielu(to_float(src[i]), a, b));
  }
}

}  // namespace

// stream [rows, cols] float32 += weight * g / sqrt(mean(g^2) + eps) with g = y * sigmoid(z + z_bias); y [rows, cols] float32, z
// [rows, cols] in z_dtype with rows of z_stride (null: g = y), z_bias float32 [cols] or null, weight float32 [cols].  normed (in
// normed_dtype, or null): the new rows over sqrt(mean(row^2) + next_eps), times next_weight (float32 [cols]).
LRS_API int lrs_gated_norm_add(float* stream_rows, const float* y, const void* z, int z_dtype, int z_stride, const float* z_bias,
                               const float* weight, float eps, int rows, int cols, const float* next_weight, float next_eps, void* normed,
                               int normed_dtype, void* stream) {
  LRS_REQUIRE(rows > 0 && cols > 0 && eps > 0.f, "gated_norm_add: bad sizes rows=%d cols=%d", rows, cols);
  LRS_REQUIRE(!z || z_stride >= cols, "gated_norm_add: gate rows of %d hold fewer than %d values", z_stride, cols);
  LRS_REQUIRE(!normed || (next_weight && next_eps > 0.f), "gated_norm_add: the norm that follows needs a weight and a positive eps");
  hipStream_t s = (hipStream_t)stream;
  const int z_item = z_dtype == LRS_F32 ? 4 : 2, n_item = normed_dtype == LRS_F32 ? 4 : 2;
  const bool vec = cols % 4 == 0 && cols <= 8192 &&
                   ((uintptr_t)stream_rows | (uintptr_t)y | (uintptr_t)z_bias | (uintptr_t)weight | (uintptr_t)next_weight) % 16 == 0 &&
                   (uintptr_t)z % (4 * z_item) == 0 && z_stride % 4 == 0 && (uintptr_t)normed % (4 * n_item) == 0;
#define ARGS(TZ, TN) stream_rows, y, (const TZ*)z, z_stride, z_bias, weight, eps, cols, next_weight, next_eps, (TN*)normed
#define PICK(TZ, TN)                                                                                                            \
  do {                                                                                                                          \
    if (vec && cols > 2048) gated_norm_add_vec_kernel<TZ, TN, 1024><<<rows, 1024, 0, s>>>(ARGS(TZ, TN));                        \
    else if (vec) gated_norm_add_vec_kernel<TZ, TN, 512><<<rows, 512, 0, s>>>(ARGS(TZ, TN));                                    \
    else gated_norm_add_kernel<TZ, TN><<<rows, 256, 0, s>>>(ARGS(TZ, TN));                                                      \
  } while (0)
  if (z_dtype == LRS_F32 && normed_dtype == LRS_F32) PICK(float, float);
  else if (z_dtype == LRS_F32 && normed_dtype == LRS_BF16) PICK(float, bf16);
  else if (z_dtype == LRS_BF16 && normed_dtype == LRS_F32) PICK(bf16, float);
  else if (z_dtype == LRS_BF16 && normed_dtype == LRS_BF16) PICK(bf16, bf16);
  else return lrs_fail("gated_norm_add: unknown dtypes %d and %d", z_dtype, normed_dtype);
#undef PICK
#undef ARGS
  return lrs_check_launch("gated_norm_add");
}

// out [rows, cols] = act(x [rows, cols]), rows of their own strides (out may be x); numbers: a and b, two float32 on the device.
LRS_API int lrs_xielu(void* out, int out_stride, const void* x, int x_stride, int dtype, int rows, int cols, const float* numbers, void* stream) {
  LRS_REQUIRE(rows > 0 && cols > 0 && out_stride >= cols && x_stride >= cols, "xielu: bad sizes rows=%d cols=%d", rows, cols);
  LRS_REQUIRE(dtype == LRS_F32 || dtype == LRS_BF16, "xielu: unknown dtype %d", dtype);
  const int run = dtype == LRS_F32 ? 4 : 8, per_row = (cols + run - 1) / run;
  const int64_t pieces = (int64_t)rows * per_row;
  const unsigned blocks = (unsigned)((pieces + 255) / 256);
  hipStream_t s = (hipStream_t)stream;
  if (dtype == LRS_F32) xielu_kernel<float><<<blocks, 256, 0, s>>>((float*)out, out_stride, (const float*)x, x_stride, pieces, per_row, cols, numbers);
  else xielu_kernel<bf16><<<blocks, 256, 0, s>>>((bf16*)out, out_stride, (const bf16*)x, x_stride, pieces, per_row, cols, numbers);
  return lrs_check_launch("xielu");
}
