// Attention heads whose q and k are normalised over the whole projection (all heads of a token at once), and the
// small elementwise kernels of layers that run their sublayers side by side.
//
//   qkv_norm_prep   per token of the fused projection row [q: nq*d | k: nkv*d | v: nkv*dv | ...]: the RMS norm of the
//                   whole q part and of the whole k part (one sum of squares each, a weight per column), the half-split
//                   rotation of the first 2*rot_half dims of every q and k head, q written back in place, k into the
//                   key pages [page, kv_head, slot, d], v into the value pages [page, kv_head, dv, slot].  On the way, where
//                   asked for: a bias per column added before anything else, the queries multiplied by a temperature that
//                   grows with the position, the values mixed with those of an earlier layer (value_pages.h);
//   sigmoid_gate    out[t, c] *= sigmoid(gate[t, c / group]): the output gate of the heads, a value a column or one a head;
//   axpby           out = alpha * a + beta * b over float32 rows: sums of sublayer outputs and the scaled residual add,
//                   optionally followed by the RMS norm of the new rows (the next layer's input) in the same pass;
//   activation      out = act(x) elementwise: exact (erf) gelu, tanh gelu, silu, relu, the square of relu.
#include "value_pages.h"

namespace {

// A query at position p is multiplied by 1 + coef * ln(floor((p + 1) / every) + 1) (every 0: by one).
struct QueryTemperature {
  const int* positions;
  float coef;
  int every;
};
__device__ __forceinline__ float temperature_of(const QueryTemperature& t, int token) {
  return t.every > 0 ? 1.f + t.coef * logf((float)((t.positions[token] + 1) / t.every) + 1.f) : 1.f;
}

template <typename T>
__global__ __launch_bounds__(256) void qkv_norm_prep_kernel(T* __restrict__ qkv, int row_stride, int nq, int nkv, int d, int dv,
                                                            const float* __restrict__ q_weight, const float* __restrict__ k_weight,
                                                            float eps, const float* __restrict__ cosv, const float* __restrict__ sinv,
                                                            int rot_half, T* __restrict__ k_pages, T* __restrict__ v_pages,
                                                            const int* __restrict__ slots, int page_size, const float* __restrict__ bias,
                                                            QueryTemperature temperature, ValuePath<T> path) {
  __shared__ float scratch[32];
  const int token = blockIdx.x, tid = threadIdx.x;
  T* row = qkv + (int64_t)token * row_stride;
  const int qn = nq * d, kn = nkv * d;
  float ssq = 0.f, ssk = 0.f;
  for (int e = tid; e < qn; e += 256) {
    const float x = to_float(row[e]) + (bias ? bias[e] : 0.f);
    ssq = fmaf(x, x, ssq);
  }
  for (int e = tid; e < kn; e += 256) {
    const float x = to_float(row[qn + e]) + (bias ? bias[qn + e] : 0.f);
    ssk = fmaf(x, x, ssk);
  }
  block_sum2(ssq, ssk, scratch);
  const float inv_q = (q_weight ? 1.0f / sqrtf(ssq / (float)qn + eps) : 1.f) * temperature_of(temperature, token);
  const float inv_k = k_weight ? 1.0f / sqrtf(ssk / (float)kn + eps) : 1.f;
  const int slot = slots ? slots[token] : -1;
  const int64_t page = slot >= 0 ? slot / page_size : 0, off = slot >= 0 ? slot % page_size : 0;
  const float* cosrow = cosv + (int64_t)token * rot_half;
  const float* sinrow = sinv + (int64_t)token * rot_half;
  // a head's work items: item j < rot_half is the pair (j, j + rot_half), item j >= rot_half the single dim j + rot_half;
  // no two items touch the same value, so q can be written where it was read
  const int items = d - rot_half;
  for (int w = tid; w < (nq + nkv) * items; w += 256) {
    const int head = w / items, j = w % items;
    const bool is_q = head < nq;
    if (!is_q && slot < 0) continue;
    const T* src = row + (int64_t)head * d;
    const float* weight = is_q ? q_weight : k_weight;
    const float* hb = bias ? bias + (int64_t)head * d : nullptr;
    const int wbase = (is_q ? head : head - nq) * d;
    const float inv = is_q ? inv_q : inv_k;
    T* dst = is_q ? row + (int64_t)head * d : k_pages + ((page * nkv + (head - nq)) * page_size + off) * d;
    if (j < rot_half) {
      float a = (to_float(src[j]) + (hb ? hb[j] : 0.f)) * inv, b = (to_float(src[j + rot_half]) + (hb ? hb[j + rot_half] : 0.f)) * inv;
      if (weight) {
        a *= weight[wbase + j];
        b *= weight[wbase + j + rot_half];
      }
      const float c = cosrow[j], s = sinrow[j];
      dst[j] = from_float<T>(a * c - b * s);
      dst[j + rot_half] = from_float<T>(b * c + a * s);
    } else {
      const int i = j + rot_half;
      float a = (to_float(src[i]) + (hb ? hb[i] : 0.f)) * inv;
      if (weight) a *= weight[wbase + i];
      dst[i] = from_float<T>(a);
    }
  }
  if (slot >= 0 && v_pages) {           // (null: values_in_runs_kernel stores them)
    store_values(path, row, qn + kn, token, nkv, dv, v_pages, page, off, page_size, tid, 256);
  }
}

// The same in bfloat16 for heads whose size and rotated half are multiples of eight and rows of q and k of up to 8,192 values:
// 16 bytes a load, a work item is a run of eight dims (with its partner eight of the other half where the head is rotated
// there), and the rows stay in registers between the sums of squares and the norms.
constexpr int PREP_ITEMS = 4;       // work items a thread holds

__global__ __launch_bounds__(256) void qkv_norm_prep_vec_kernel(bf16* __restrict__ qkv, int row_stride, int nq, int nkv, int d, int dv,
                                                                const float* __restrict__ q_weight, const float* __restrict__ k_weight,
                                                                float eps, const float* __restrict__ cosv, const float* __restrict__ sinv,
                                                                int rot_half, bf16* __restrict__ k_pages, bf16* __restrict__ v_pages,
                                                                const int* __restrict__ slots, int page_size, const float* __restrict__ bias,
                                                                QueryTemperature temperature, ValuePath<bf16> path) {
  __shared__ float scratch[32];
  const int token = blockIdx.x, tid = threadIdx.x;
  bf16* row = qkv + (int64_t)token * row_stride;
  const int qn = nq * d, kn = nkv * d;
  const int rot8 = rot_half / 8, items = (d - rot_half) / 8, total = (nq + nkv) * items;
  bf16x8 lo[PREP_ITEMS], hi[PREP_ITEMS];
  // eight values of a run with their biases added (asked for twice, for the sum of squares and for the write: the same bits)
  auto biased = [&](const bf16x8& x, const float* b, float (&out)[8]) {
    floatx4 b0 = {0.f, 0.f, 0.f, 0.f}, b1 = b0;
    if (b) b0 = *(const floatx4*)b, b1 = *(const floatx4*)(b + 4);
#pragma unroll
    for (int i = 0; i < 8; ++i) out[i] = (float)x[i] + (i < 4 ? b0[i] : b1[i - 4]);
  };
  const int slot = slots ? slots[token] : -1;
  const int64_t page = slot >= 0 ? slot / page_size : 0, off = slot >= 0 ? slot % page_size : 0;
  // (the values need no sum: theirs are on their way while the others' are made)
  if (slot >= 0 && v_pages) {           // (null: values_in_runs_kernel stores them)
    store_values(path, row, qn + kn, token, nkv, dv, v_pages, page, off, page_size, tid, 256);
  }
  float ssq = 0.f, ssk = 0.f;
#pragma unroll
  for (int n = 0; n < PREP_ITEMS; ++n) {
    const int w = tid + n * 256;
    if (w < total) {
      const int head = w / items, j = w % items;
      const bf16* src = row + (int64_t)head * d;
      const float* hb = bias ? bias + (int64_t)head * d : nullptr;
      const bool paired = j < rot8;
      const int at = paired ? j * 8 : j * 8 + rot_half;
      lo[n] = *(const bf16x8*)(src + at);
      float ss = 0.f, x[8];
      biased(lo[n], hb ? hb + at : nullptr, x);
#pragma unroll
      for (int i = 0; i < 8; ++i) ss = fmaf(x[i], x[i], ss);
      if (paired) {
        hi[n] = *(const bf16x8*)(src + j * 8 + rot_half);
        biased(hi[n], hb ? hb + j * 8 + rot_half : nullptr, x);
#pragma unroll
        for (int i = 0; i < 8; ++i) ss = fmaf(x[i], x[i], ss);
      }
      if (head < nq) ssq += ss;
      else ssk += ss;
    }
  }
  block_sum2(ssq, ssk, scratch);
  const float inv_q = (q_weight ? 1.0f / sqrtf(ssq / (float)qn + eps) : 1.f) * temperature_of(temperature, token);
  const float inv_k = k_weight ? 1.0f / sqrtf(ssk / (float)kn + eps) : 1.f;
  const float* cosrow = cosv + (int64_t)token * rot_half;
  const float* sinrow = sinv + (int64_t)token * rot_half;
#pragma unroll
  for (int n = 0; n < PREP_ITEMS; ++n) {
    const int w = tid + n * 256;
    if (w >= total) continue;
    const int head = w / items, j = w % items;
    const bool is_q = head < nq;
    if (!is_q && slot < 0) continue;
    const float* weight = is_q ? q_weight : k_weight;
    const int wbase = (is_q ? head : head - nq) * d;
    const float inv = is_q ? inv_q : inv_k;
    bf16* dst = is_q ? row + (int64_t)head * d : k_pages + ((page * nkv + (head - nq)) * page_size + off) * d;
    const floatx4 one4 = {1.f, 1.f, 1.f, 1.f};
    const float* hb = bias ? bias + (int64_t)head * d : nullptr;
    float xl[8], xh[8];
    biased(lo[n], hb ? hb + (j < rot8 ? j * 8 : j * 8 + rot_half) : nullptr, xl);
    if (j < rot8) {
      biased(hi[n], hb ? hb + j * 8 + rot_half : nullptr, xh);
      // weights and angles of the eight pairs, 16 bytes a load, all asked for before any is used
      floatx4 wa[2], wb[2], c4[2], s4[2];
#pragma unroll
      for (int half = 0; half < 2; ++half) {
        wa[half] = weight ? *(const floatx4*)(weight + wbase + j * 8 + half * 4) : one4;
        wb[half] = weight ? *(const floatx4*)(weight + wbase + j * 8 + rot_half + half * 4) : one4;
        c4[half] = *(const floatx4*)(cosrow + j * 8 + half * 4);
        s4[half] = *(const floatx4*)(sinrow + j * 8 + half * 4);
      }
      bf16x8 first, second;
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        const float a = xl[i] * inv * wa[i / 4][i % 4], b = xh[i] * inv * wb[i / 4][i % 4];
        const float c = c4[i / 4][i % 4], sn = s4[i / 4][i % 4];
        first[i] = (bf16)(a * c - b * sn);
        second[i] = (bf16)(b * c + a * sn);
      }
      *(bf16x8*)(dst + j * 8) = first;
      *(bf16x8*)(dst + j * 8 + rot_half) = second;
    } else {
      const int at = j * 8 + rot_half;
      floatx4 wa[2];
#pragma unroll
      for (int half = 0; half < 2; ++half) wa[half] = weight ? *(const floatx4*)(weight + wbase + at + half * 4) : one4;
      bf16x8 only;
#pragma unroll
      for (int i = 0; i < 8; ++i) only[i] = (bf16)(xl[i] * inv * wa[i / 4][i % 4]);
      *(bf16x8*)(dst + at) = only;
    }
  }
}

template <typename T>
__global__ void sigmoid_gate_kernel(T* __restrict__ out, int out_stride, const T* __restrict__ gate, int gate_stride, int rows, int cols,
                                    int group) {
  const int64_t e = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (e >= (int64_t)rows * cols) return;
  const int64_t r = e / cols, c = e % cols;
  const float g = to_float(gate[r * gate_stride + c / group]);     // one gate value for every `group` neighbouring columns
  T* o = out + r * out_stride + c;
  *o = from_float<T>(to_float(*o) / (1.f + expf(-g)));
}

__global__ void axpby_kernel(float* __restrict__ out, const float* __restrict__ a, float alpha, const float* __restrict__ b, float beta,
                             int64_t count) {
  const int64_t e = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (e < count) out[e] = alpha * a[e] + beta * b[e];
}

// out = alpha * a + beta * b for one row a workgroup, and the row's RMS norm times a weight beside it.
template <typename TN>
__global__ __launch_bounds__(256) void axpby_norm_kernel(float* __restrict__ out, const float* __restrict__ a, float alpha,
                                                         const float* __restrict__ b, float beta, int cols,
                                                         const float* __restrict__ norm_weight, float eps, TN* __restrict__ normed) {
  __shared__ float scratch[16];
  const int64_t base = (int64_t)blockIdx.x * cols;
  float ss = 0.f;
  for (int c = threadIdx.x; c < cols; c += 256) {
    const float v = alpha * a[base + c] + beta * b[base + c];
    out[base + c] = v;
    ss = fmaf(v, v, ss);
  }
  ss = block_sum(ss, scratch);
  const float inv = 1.0f / sqrtf(ss / (float)cols + eps);
  for (int c = threadIdx.x; c < cols; c += 256) normed[base + c] = from_float<TN>(out[base + c] * inv * norm_weight[c]);
}

// The same for rows of up to 8,192 values, a multiple of four: 16 bytes a load, the row stays in registers between the sum of
// squares and the norm, and every load is on its way before the first is used.
template <typename TN>
__global__ __launch_bounds__(256) void axpby_norm_vec_kernel(float* __restrict__ out, const float* __restrict__ a, float alpha,
                                                             const float* __restrict__ b, float beta, int cols,
                                                             const float* __restrict__ norm_weight, float eps, TN* __restrict__ normed) {
  constexpr int PER = 8;
  __shared__ float scratch[16];
  const int64_t base = (int64_t)blockIdx.x * cols;
  const int quads = cols / 4;
  floatx4 va[PER], vb[PER], w[PER];
#pragma unroll
  for (int n = 0; n < PER; ++n) {
    const int q = threadIdx.x + n * 256;
    if (q < quads) {
      va[n] = *(const floatx4*)(a + base + 4 * q);
      vb[n] = *(const floatx4*)(b + base + 4 * q);
      w[n] = *(const floatx4*)(norm_weight + 4 * q);
    }
  }
  float ss = 0.f;
#pragma unroll
  for (int n = 0; n < PER; ++n) {
    const int q = threadIdx.x + n * 256;
    if (q < quads) {
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        va[n][i] = alpha * va[n][i] + beta * vb[n][i];
        ss = fmaf(va[n][i], va[n][i], ss);
      }
      *(floatx4*)(out + base + 4 * q) = va[n];
    }
  }
  ss = block_sum(ss, scratch);
  const float inv = 1.0f / sqrtf(ss / (float)cols + eps);
#pragma unroll
  for (int n = 0; n < PER; ++n) {
    const int q = threadIdx.x + n * 256;
    if (q < quads) {
      TN packed[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) packed[i] = from_float<TN>(va[n][i] * inv * w[n][i]);
      if constexpr (sizeof(TN) == 4) *(floatx4*)(normed + base + 4 * q) = *(const floatx4*)packed;
      else *(uint64_t*)(normed + base + 4 * q) = *(const uint64_t*)packed;
    }
  }
}

enum { ACT_GELU_ERF = 0, ACT_GELU_TANH = 1, ACT_SILU = 2, ACT_RELU = 3, ACT_RELU_SQUARE = 4 };

__device__ __forceinline__ float activate(float x, int kind) {
  switch (kind) {
    case ACT_GELU_ERF: return 0.5f * x * (1.f + erff(x * 0.70710678118654752f));
    case ACT_GELU_TANH: return 0.5f * x * (1.f + tanhf(0.7978845608028654f * (x + 0.044715f * x * x * x)));
    case ACT_SILU: return x / (1.f + expf(-x));
    case ACT_RELU_SQUARE: return x > 0.f ? x * x : 0.f;
    default: return fmaxf(x, 0.f);
  }
}

template <typename T>
__global__ void activation_kernel(T* __restrict__ out, const T* __restrict__ x, int64_t count, int kind) {
  const int64_t e = (int64_t)blockIdx.x * blockDim.x + threadIdx.x;
  if (e < count) out[e] = from_float<T>(activate(to_float(x[e]), kind));
}

// The same 16 bytes at a time, for counts that are a multiple of that.
template <typename T, int KIND>
__global__ __launch_bounds__(256) void activation_vec_kernel(T* __restrict__ out, const T* __restrict__ x, int64_t pieces) {
  constexpr int RUN = 16 / sizeof(T);
  typedef T vec __attribute__((ext_vector_type(RUN)));
  const int64_t e = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (e >= pieces) return;
  vec v = ((const vec*)x)[e];
#pragma unroll
  for (int i = 0; i < RUN; ++i) v[i] = from_float<T>(activate(to_float(v[i]), KIND));
  ((vec*)out)[e] = v;
}

}  // namespace

// qkv [tokens, row_stride] in dtype: q (nq*d) | k (nkv*d) | v (nkv*dv) | anything else.  q_weight [nq*d], k_weight [nkv*d]
// float32 (both null: no norm).  cos, sin [tokens, rot_half] float32.  slots[t] = page * page_size + offset (negative: the
// token's key and value are not stored).  bias (float32 [nq*d + nkv*d + nkv*dv], or null) is added to q, k and v as they are read.
// every > 0: queries are multiplied by 1 + coef * ln(floor((positions[t] + 1) / every) + 1).  first_values [tokens, nkv*dv] in
// dtype, or null: value_mix null leaves the step's values there, value_mix given (one float32 on the device) mixes
// v <- (1 - value_mix) v + value_mix first_values.  nq may be 0 (rows that begin with the key heads: queries that stay as they are).
LRS_API int lrs_qkv_norm_prep(void* qkv, int dtype, int tokens, int row_stride, int nq, int nkv, int d, int dv, const float* q_weight,
                              const float* k_weight, float eps, const float* cosv, const float* sinv, int rot_half, void* k_pages,
                              void* v_pages, const int* slots, int page_size, const float* bias, const int* positions, float coef, int every,
                              void* first_values, const float* value_mix, void* stream) {
  LRS_REQUIRE(tokens > 0 && nq >= 0 && nkv > 0 && d > 0 && dv > 0, "qkv_norm_prep: bad sizes tokens=%d nq=%d nkv=%d d=%d dv=%d", tokens, nq, nkv, d, dv);
  LRS_REQUIRE(row_stride >= nq * d + nkv * d + nkv * dv, "qkv_norm_prep: rows of %d hold fewer than q, k and v", row_stride);
  LRS_REQUIRE(rot_half >= 0 && 2 * rot_half <= d, "qkv_norm_prep: rotary width %d exceeds head_dim %d", 2 * rot_half, d);
  LRS_REQUIRE(rot_half == 0 || (cosv && sinv), "qkv_norm_prep: rotation asked for without tables");
  LRS_REQUIRE((q_weight == nullptr) == (k_weight == nullptr), "qkv_norm_prep: q and k norm weights must come together");
  LRS_REQUIRE(!q_weight || (eps > 0.f && nq > 0), "qkv_norm_prep: eps must be positive, and norms come with query heads");
  LRS_REQUIRE(k_pages && v_pages && slots && page_size > 0, "qkv_norm_prep: cache write needs pages, slots and a page size");
  LRS_REQUIRE(every >= 0 && (every == 0 || positions), "qkv_norm_prep: a temperature needs a positive step and the positions");
  LRS_REQUIRE(!value_mix || first_values, "qkv_norm_prep: nothing to mix the values with");
  hipStream_t s = (hipStream_t)stream;
  const QueryTemperature temperature{positions, coef, every};
  // steps of many tokens: the values as runs of slots, 16 bytes a store, by workgroups of their own (token by token they are
  // 2-byte writes a page row apart)
  if (tokens >= 64 && page_size % (dtype == LRS_F32 ? 4 : 8) == 0 && (uintptr_t)v_pages % 16 == 0) {
    const dim3 vgrid((tokens + 15) / 16, nkv);
    if (dtype == LRS_F32)
      values_in_runs_kernel<float><<<vgrid, 256, 0, s>>>((const float*)qkv, row_stride, (nq + nkv) * d, tokens, nkv, dv, (float*)v_pages, slots, page_size,
                                                         ValuePath<float>{bias, (float*)first_values, value_mix});
    else if (dtype == LRS_BF16)
      values_in_runs_kernel<bf16><<<vgrid, 256, 0, s>>>((const bf16*)qkv, row_stride, (nq + nkv) * d, tokens, nkv, dv, (bf16*)v_pages, slots, page_size,
                                                        ValuePath<bf16>{bias, (bf16*)first_values, value_mix});
    else return lrs_fail("qkv_norm_prep: unknown dtype %d", dtype);
    if (lrs_check_launch("values_in_runs")) return 1;
    v_pages = nullptr;
  }
  if (dtype == LRS_F32)
    qkv_norm_prep_kernel<float><<<tokens, 256, 0, s>>>((float*)qkv, row_stride, nq, nkv, d, dv, q_weight, k_weight, eps, cosv, sinv, rot_half,
                                                       (float*)k_pages, (float*)v_pages, slots, page_size, bias, temperature,
                                                       ValuePath<float>{bias, (float*)first_values, value_mix});
  else if (dtype == LRS_BF16 && d % 8 == 0 && rot_half % 8 == 0 && row_stride % 8 == 0 &&
           ((uintptr_t)qkv | (uintptr_t)q_weight | (uintptr_t)k_weight | (uintptr_t)cosv | (uintptr_t)sinv | (uintptr_t)bias | (uintptr_t)k_pages) % 16 == 0 &&
           (nq + nkv) * (d - rot_half) / 8 <= 256 * PREP_ITEMS)
    qkv_norm_prep_vec_kernel<<<tokens, 256, 0, s>>>((bf16*)qkv, row_stride, nq, nkv, d, dv, q_weight, k_weight, eps, cosv, sinv, rot_half,
                                                    (bf16*)k_pages, (bf16*)v_pages, slots, page_size, bias, temperature,
                                                    ValuePath<bf16>{bias, (bf16*)first_values, value_mix});
  else if (dtype == LRS_BF16)
    qkv_norm_prep_kernel<bf16><<<tokens, 256, 0, s>>>((bf16*)qkv, row_stride, nq, nkv, d, dv, q_weight, k_weight, eps, cosv, sinv, rot_half,
                                                      (bf16*)k_pages, (bf16*)v_pages, slots, page_size, bias, temperature,
                                                      ValuePath<bf16>{bias, (bf16*)first_values, value_mix});
  else return lrs_fail("qkv_norm_prep: unknown dtype %d", dtype);
  return lrs_check_launch("qkv_norm_prep");
}

LRS_API int lrs_sigmoid_gate(void* out, int out_stride, const void* gate, int gate_stride, int dtype, int rows, int cols, int group, void* stream) {
  LRS_REQUIRE(rows > 0 && cols > 0 && group > 0 && cols % group == 0 && out_stride >= cols && gate_stride >= cols / group,
              "sigmoid_gate: bad sizes rows=%d cols=%d group=%d", rows, cols, group);
  const int64_t count = (int64_t)rows * cols;
  const unsigned blocks = (unsigned)((count + 255) / 256);
  hipStream_t s = (hipStream_t)stream;
  if (dtype == LRS_F32) sigmoid_gate_kernel<float><<<blocks, 256, 0, s>>>((float*)out, out_stride, (const float*)gate, gate_stride, rows, cols, group);
  else if (dtype == LRS_BF16) sigmoid_gate_kernel<bf16><<<blocks, 256, 0, s>>>((bf16*)out, out_stride, (const bf16*)gate, gate_stride, rows, cols, group);
  else return lrs_fail("sigmoid_gate: unknown dtype %d", dtype);
  return lrs_check_launch("sigmoid_gate");
}

// out = alpha * a + beta * b, float32 [rows, cols] contiguous (out may be a or b).  norm_weight given: normed [rows, cols] in
// normed_dtype receives out / sqrt(mean(out^2) + eps) * norm_weight as well.
LRS_API int lrs_axpby(float* out, const float* a, float alpha, const float* b, float beta, int rows, int cols, const float* norm_weight,
                      float eps, void* normed, int normed_dtype, void* stream) {
  LRS_REQUIRE(rows > 0 && cols > 0, "axpby: bad sizes rows=%d cols=%d", rows, cols);
  hipStream_t s = (hipStream_t)stream;
  if (norm_weight == nullptr) {
    const int64_t count = (int64_t)rows * cols;
    axpby_kernel<<<(unsigned)((count + 255) / 256), 256, 0, s>>>(out, a, alpha, b, beta, count);
  } else {
    LRS_REQUIRE(normed && eps > 0.f, "axpby: the norm needs a buffer and a positive eps");
    const bool vec = cols % 4 == 0 && cols <= 8192 && ((uintptr_t)out | (uintptr_t)a | (uintptr_t)b | (uintptr_t)norm_weight | (uintptr_t)normed) % 16 == 0;
    if (normed_dtype == LRS_F32 && vec) axpby_norm_vec_kernel<float><<<rows, 256, 0, s>>>(out, a, alpha, b, beta, cols, norm_weight, eps, (float*)normed);
    else if (normed_dtype == LRS_BF16 && vec) axpby_norm_vec_kernel<bf16><<<rows, 256, 0, s>>>(out, a, alpha, b, beta, cols, norm_weight, eps, (bf16*)normed);
    else if (normed_dtype == LRS_F32) axpby_norm_kernel<float><<<rows, 256, 0, s>>>(out, a, alpha, b, beta, cols, norm_weight, eps, (float*)normed);
    else if (normed_dtype == LRS_BF16) axpby_norm_kernel<bf16><<<rows, 256, 0, s>>>(out, a, alpha, b, beta, cols, norm_weight, eps, (bf16*)normed);
    else return lrs_fail("axpby: unknown dtype %d", normed_dtype);
  }
  return lrs_check_launch("axpby");
}

LRS_API int lrs_activation(void* out, const void* x, int dtype, int64_t count, int kind, void* stream) {
  LRS_REQUIRE(count > 0 && kind >= 0 && kind <= ACT_RELU_SQUARE, "activation: bad arguments count=%lld kind=%d", (long long)count, kind);
  const unsigned blocks = (unsigned)((count + 255) / 256);
  hipStream_t s = (hipStream_t)stream;
  const int run = dtype == LRS_F32 ? 4 : 8;
  if ((dtype == LRS_F32 || dtype == LRS_BF16) && count % run == 0 && ((uintptr_t)out | (uintptr_t)x) % 16 == 0) {
    const int64_t pieces = count / run;
    const unsigned grid = (unsigned)((pieces + 255) / 256);
#define VEC(KIND)                                                                                                               \
  case KIND:                                                                                                                    \
    if (dtype == LRS_F32) activation_vec_kernel<float, KIND><<<grid, 256, 0, s>>>((float*)out, (const float*)x, pieces);        \
    else activation_vec_kernel<bf16, KIND><<<grid, 256, 0, s>>>((bf16*)out, (const bf16*)x, pieces);                            \
    break
    switch (kind) {
      VEC(ACT_GELU_ERF);
      VEC(ACT_GELU_TANH);
      VEC(ACT_SILU);
      VEC(ACT_RELU);
      VEC(ACT_RELU_SQUARE);
    }
#undef VEC
    return lrs_check_launch("activation");
  }
  if (dtype == LRS_F32) activation_kernel<float><<<blocks, 256, 0, s>>>((float*)out, (const float*)x, count, kind);
  else if (dtype == LRS_BF16) activation_kernel<bf16><<<blocks, 256, 0, s>>>((bf16*)out, (const bf16*)x, count, kind);
  else return lrs_fail("activation: unknown dtype %d", dtype);
  return lrs_check_launch("activation");
}
