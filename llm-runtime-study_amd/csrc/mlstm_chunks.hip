// The matrix memory with exponential gates (delta.hip, mLSTM) over long portions in bfloat16 runs: chunks of 64 tokens on the
// matrix cores, the state carried from chunk to chunk in float32.
//
// Within a chunk let F_t be the sum of the log forget gates up to token t and J_s = i_s - F_s.  With m0, S0 from the chunk before,
//     m_t = max(m0 + F_t, mu_t),  mu_t = F_t + max_{s <= t} J_s
//     o_t ~ exp(m0 + F_t - m_t) S0^T q_t + exp(mu_t - m_t) sum_{s <= t} P_ts v_s,   P_ts = exp(F_t + J_s - mu_t) (q_t . k_s)
//     S_L = exp(m0 + F_L - m_L) S0 + sum_s exp(F_L + J_s - m_L) k_s v_s^T
// (every exponent is at most zero; the normaliser n is a column of S whose values are one, as in the scan).  mu and P need nothing
// of the chunks before, so
//   mlstm_pack    per (chunk, head), all chunks at once: the gates, P, and q and k as operands of the products;
//   mlstm_chunks  per (request, head, 16 or 32 columns of S): walks the chunks with its part of S in accumulators.
// Precision: q, k and v are what a bfloat16 run's projections are, rounded once, and exact operands; P, the state as an operand and the
// weighted values are split into two bfloat16 numbers each (their sum is good to 2^-17 of the value) and multiplied in two products;
// sums, the state itself and everything about the gates are float32.
#include "common.h"

int lrs_mlstm_read_out(void* out, int out_dtype, const float* raw, const float* floors, const float* proj, int ld, int g_at, const float* norm_w,
                       float q_factor, float eps, int tokens, int requests, int H, int dv, const float* maxima, const int* token_request, const int* cu,
                       const int* slot_ids, float* state, int64_t state_stride, int64_t m_offset, hipStream_t s);
void lrs_mlstm_singles(const float* proj, int ld, int requests, const int* slot_ids, float* state, int64_t state_stride, int H, int d, int dv,
                       const float* i_bias, const float* f_bias, float cap, float* raw, float* floors, float* maxima, hipStream_t s);
extern "C" int lrs_delta_state_rows(int d);

namespace {

constexpr int L = 64;             // tokens of a chunk: one a lane where the gates are worked out
constexpr int SPLIT = 16;         // lanes of a column in the state row's layout (delta.hip)

// A request's chunks lie side by side in the packs: request r's chunk c in slot cu[r] / L + r + c (requests never share one).
__device__ __forceinline__ int first_slot(const int* __restrict__ cu, int r) { return cu[r] / L + r; }

__device__ __forceinline__ void split_bf16(float x, bf16& hi, bf16& lo) {
  hi = (bf16)x;
  lo = (bf16)(x - (float)hi);
}

// The packs hold operands in the order in which a wave's lanes take them: of every 16 rows and 32 columns of the product, row
// r's eight columns 8 g .. 8 g + 7 are lane 16 g + r's 16 bytes, so that a load is 1,024 bytes in a row.
__device__ __forceinline__ int fragment(int rows16, int steps, int step, int row, int g) { return ((rows16 * steps + step) * WAVE + g * 16 + row) * 8; }

// q_pack [slot, H, L, DP], k_pack [slot, H, DP, L], p_pack [slot, H, 2, L, L] (the two halves of P, [t][s]), each in fragments,
// gate_pack [slot, H, 3, L]: F, J, mu (tokens past the request's end: F and mu of its last token, J -inf, q, k and P zero).
template <int DP>
__global__ __launch_bounds__(256) void mlstm_pack_kernel(const float* __restrict__ proj, int ld, int k_at, int i_at, int f_at,
                                                         const float* __restrict__ i_bias, const float* __restrict__ f_bias, float cap,
                                                         const int* __restrict__ cu, int requests, int H, int d, bf16* __restrict__ q_pack,
                                                         bf16* __restrict__ k_pack, bf16* __restrict__ p_pack, float* __restrict__ gate_pack) {
  constexpr int LD = DP + 16;      // rows 32 bytes more than a multiple of 64 apart: 16-byte reads of 16 rows at the full rate
  __shared__ __attribute__((aligned(16))) bf16 qs[L * LD];
  __shared__ __attribute__((aligned(16))) bf16 ks[L * LD];
  __shared__ float f_sum[L], j_of[L], mu_of[L];
  const int slot = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid % WAVE, wave = tid / WAVE;
  // the request whose chunk this slot is: the last one that begins at or before it
  int r = -1;
  for (int r0 = 0; r0 < requests; r0 += WAVE) {
    const bool before = r0 + lane < requests && first_slot(cu, r0 + lane) <= slot;
    r += __popcll(__ballot(before));
  }
  if (r < 0) return;
  const int chunk = slot - first_slot(cu, r), n = cu[r + 1] - cu[r];
  if (chunk * L >= n) return;
  const int token0 = cu[r] + chunk * L, count = min(L, n - chunk * L);
  const int64_t pack = (int64_t)slot * H + h;

  if (wave == 0) {
    const int64_t token = token0 + min(lane, count - 1);
    const float yi = cap * tanhf((proj[token * ld + i_at + h] + i_bias[h]) / cap), yf = cap * tanhf((proj[token * ld + f_at + h] + f_bias[h]) / cap);
    float f = lane < count ? fminf(yf, 0.f) - log1pf(expf(-fabsf(yf))) : 0.f;
#pragma unroll
    for (int step = 1; step < WAVE; step *= 2) {          // sums over the lanes up to this one
      const float other = __shfl_up(f, step, WAVE);
      if (lane >= step) f += other;
    }
    const float j = lane < count ? yi - f : -INFINITY;
    float top = j;
#pragma unroll
    for (int step = 1; step < WAVE; step *= 2) {
      const float other = __shfl_up(top, step, WAVE);
      if (lane >= step) top = fmaxf(top, other);
    }
    float* g = gate_pack + pack * 3 * L;
    g[lane] = f_sum[lane] = f;
    g[L + lane] = j_of[lane] = j;
    g[2 * L + lane] = mu_of[lane] = f + top;
  }

  // q and k, rounded: rows into LDS, q's rows into its pack as well; four values a piece
  const bool whole = d % 4 == 0 && ld % 4 == 0 && k_at % 4 == 0;
  for (int e = tid; e < L * DP / 4; e += 256) {
    const int t = e / (DP / 4), i = e % (DP / 4) * 4;
    float a[4] = {0.f, 0.f, 0.f, 0.f}, b[4] = {0.f, 0.f, 0.f, 0.f};
    if (t < count && i < d) {
      const float* row = proj + (int64_t)(token0 + t) * ld + h * d + i;
      if (whole) {
        const floatx4 qa = *(const floatx4*)row, kb = *(const floatx4*)(row + k_at);
#pragma unroll
        for (int x = 0; x < 4; ++x) a[x] = qa[x], b[x] = kb[x];
      } else {
        for (int x = 0; x < 4; ++x)
          if (i + x < d) a[x] = row[x], b[x] = row[k_at + x];
      }
    }
    const bf16x4 qa = {(bf16)a[0], (bf16)a[1], (bf16)a[2], (bf16)a[3]}, kb = {(bf16)b[0], (bf16)b[1], (bf16)b[2], (bf16)b[3]};
    *(bf16x4*)(qs + t * LD + i) = qa;
    *(bf16x4*)(ks + t * LD + i) = kb;
    *(bf16x4*)(q_pack + pack * L * DP + fragment(t / 16, DP / 32, i / 32, t % 16, i % 32 / 8) + i % 8) = qa;
  }
  __syncthreads();

  // P, a wave 16 of the t: the products come out with t in the lanes' columns and four consecutive s a lane
  {
    const int col = lane & 15, g = lane >> 4, t = wave * 16 + col;
    bf16x8 qf[DP / 32];
#pragma unroll
    for (int c = 0; c < DP / 32; ++c) qf[c] = *(const bf16x8*)(qs + t * LD + c * 32 + g * 8);
    const float ft = f_sum[t] - mu_of[t];
    bf16* hi_pack = p_pack + pack * 2 * L * L;
    bf16* lo_pack = hi_pack + L * L;
    for (int b = 0; b <= (wave | 1); ++b) {               // (whole pairs of blocks: what the second product reads at a time)
      floatx4 acc = {0.f, 0.f, 0.f, 0.f};
      if (b <= wave) {
#pragma unroll
        for (int c = 0; c < DP / 32; ++c)
          acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*(const bf16x8*)(ks + (b * 16 + col) * LD + c * 32 + g * 8), qf[c], acc, 0, 0, 0);
      }
      bf16x4 hi, lo;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int s = b * 16 + g * 4 + i;
        const float p = s <= t ? expf(ft + j_of[s]) * acc[i] : 0.f;
        bf16 ph, pl;
        split_bf16(p, ph, pl);
        hi[i] = ph, lo[i] = pl;
      }
      const int s0 = b * 16 + g * 4, at = fragment(wave, 2, s0 / 32, col, s0 % 32 / 8) + s0 % 8;
      *(bf16x4*)(hi_pack + at) = hi;
      *(bf16x4*)(lo_pack + at) = lo;
    }
  }
  // k by columns: eight tokens of a dim in one store
  for (int e = tid; e < DP * (L / 8); e += 256) {
    const int i = e % 16 + e / 64 / 2 * 16, x = e / 64 % 2, piece = e / 16 % 4, j = x * 32 + piece * 8;      // (in the order of the pack: whole lines)
    bf16x8 v;
#pragma unroll
    for (int y = 0; y < 8; ++y) v[y] = ks[(j + y) * LD + i];
    *(bf16x8*)(k_pack + pack * DP * L + fragment(i / 16, 2, x, i % 16, piece)) = v;
  }
}

// A workgroup owns C = 16 * CB columns of one head's S (dv values and the normaliser, `columns` in all) for one request, four waves
// every 16 columns.  Per chunk: S goes into LDS as two bfloat16 halves, the columns' values as they are and weighted (two halves);
// the quarter w of a column block's waves makes the read-outs of tokens 16 w .. 16 w + 15 and updates the rows of S of its DP / 64
// blocks of 16.  The operands that a wave has for itself (its rows of q, P and k) come straight from the packs, the next chunk's on
// their way while this one is worked on.
template <int DP, int CB>
__global__ __launch_bounds__(256 * CB, 2) void mlstm_chunks_kernel(const float* __restrict__ proj, int ld, int v_at, const bf16* __restrict__ q_pack,
                                                              const bf16* __restrict__ k_pack, const bf16* __restrict__ p_pack,
                                                              const float* __restrict__ gate_pack, const int* __restrict__ cu,
                                                              const int* __restrict__ slot_ids, float* __restrict__ state, int64_t state_stride,
                                                              int64_t m_offset, int H, int columns, float* __restrict__ raw,
                                                              float* __restrict__ floors, float* __restrict__ maxima) {
  constexpr int C = 16 * CB, ROWS = DP / 16, QK = DP / 32, DB = DP / 64, SLD = DP + 16, VLD = L + 16, FLD = DP + 4;
  constexpr int THREADS = 256 * CB, TOKENS = 4;            // a thread brings in the values of so many tokens of one column
  constexpr int HALVES = 2 * C * SLD * 2, PLAIN = C * FLD * 4;
  __shared__ __attribute__((aligned(16))) unsigned char s_room[HALVES > PLAIN ? HALVES : PLAIN];
  __shared__ __attribute__((aligned(16))) bf16 v_t[3][C * VLD];    // the values, the weighted values' first and second halves: [column][token]
  __shared__ __attribute__((aligned(16))) float of_state[L], of_chunk[L];               // what a token's two sums are multiplied by
  bf16* s_hi = (bf16*)s_room;
  bf16* s_lo = s_hi + C * SLD;
  float* s_f32 = (float*)s_room;
  typedef bf16 run_t __attribute__((ext_vector_type(TOKENS)));
  const int r = blockIdx.x, h = blockIdx.y, c0 = blockIdx.z * C, tid = threadIdx.x, lane = tid % WAVE;
  const int wave = tid / WAVE % 4, block = tid / WAVE / 4; // the quarter and the column block of this wave
  const int col = lane & 15, g = lane >> 4, c = block * 16 + col;
  const int start = cu[r], n = cu[r + 1] - start, chunks = (n + L - 1) / L, slot0 = first_slot(cu, r);
  float* own = state + (int64_t)slot_ids[r] * state_stride;
  float* st = own + (int64_t)h * ROWS * columns * SPLIT;
  float m = own[m_offset + h];

  // S from the state row, whose lines run over columns and 16ths of the rows, through LDS into the accumulators' layout
  for (int e = tid; e < ROWS * C * SPLIT; e += THREADS) {
    const int row = e / (C * SPLIT), cc = e / SPLIT % C, s = e % SPLIT;
    s_f32[cc * FLD + s * ROWS + row] = c0 + cc < columns ? st[((int64_t)row * columns + c0 + cc) * SPLIT + s] : 0.f;
  }
  __syncthreads();
  floatx4 S[DB];
#pragma unroll
  for (int b = 0; b < DB; ++b) S[b] = *(const floatx4*)(s_f32 + c * FLD + (wave * DB + b) * 16 + g * 4);
  __syncthreads();

  const int vc = tid % C, vt0 = tid / C * TOKENS;          // the column and the first token of the values a thread brings in
  const int values = columns - 1;
  // What a wave has on its way: every operand of the next chunk is asked for as soon as this chunk's has been used (no second set of
  // registers), without a branch around a load (behind one, every use would have to wait for all loads): past the end, of the
  // portion or of the values, any number will do and is not used.
  bf16x8 q[QK], p[2][2], k[DB][2];
  float v[TOKENS], f, mu, f_last, mu_last;
  floatx4 j;
  auto pack_of = [&](int chunk) { return (int64_t)(slot0 + min(chunk, chunks - 1)) * H + h; };
  auto fetch_values = [&](int chunk) {
    chunk = min(chunk, chunks - 1);
    const int count = min(L, n - chunk * L);
    const float* gates = gate_pack + pack_of(chunk) * 3 * L;
    const float* from = proj + (int64_t)(start + chunk * L) * ld + v_at + (int64_t)h * values + min(c0 + vc, values - 1);
#pragma unroll
    for (int x = 0; x < TOKENS; ++x) v[x] = from[(int64_t)min(vt0 + x, count - 1) * ld];
    j = *(const floatx4*)(gates + L + vt0);
    f = gates[lane], mu = gates[2 * L + lane];
    f_last = gates[L - 1], mu_last = gates[3 * L - 1];
  };
  auto fetch_q = [&](int chunk) {
    const bf16* from = q_pack + pack_of(chunk) * L * DP + lane * 8;
#pragma unroll
    for (int x = 0; x < QK; ++x) q[x] = *(const bf16x8*)(from + fragment(wave, QK, x, 0, 0));
  };
  auto fetch_p = [&](int chunk) {
    const bf16* from = p_pack + pack_of(chunk) * 2 * L * L + lane * 8;
#pragma unroll
    for (int half = 0; half < 2; ++half)
#pragma unroll
      for (int x = 0; x < 2; ++x) p[half][x] = *(const bf16x8*)(from + half * L * L + fragment(wave, 2, x, 0, 0));
  };
  auto fetch_k = [&](int chunk) {
    const bf16* from = k_pack + pack_of(chunk) * DP * L + lane * 8;
#pragma unroll
    for (int b = 0; b < DB; ++b)
#pragma unroll
      for (int x = 0; x < 2; ++x) k[b][x] = *(const bf16x8*)(from + fragment(wave * DB + b, 2, x, 0, 0));
  };
  fetch_values(0);
  fetch_q(0);
  fetch_p(0);
  fetch_k(0);
  for (int chunk = 0; chunk < chunks; ++chunk) {
    const int count = min(L, n - chunk * L);
    const float m_last = fmaxf(m + f_last, mu_last);
    float floor_here = 0.f;
    if (tid < L) {
      const float mt = fmaxf(m + f, mu);
      of_state[lane] = expf(m + f - mt);
      of_chunk[lane] = expf(mu - mt);
      floor_here = expf(-mt);
    }
    {
      run_t plain, hi, lo;
#pragma unroll
      for (int x = 0; x < TOKENS; ++x) {
        const bf16 value = (bf16)(vt0 + x < count && c0 + vc < columns ? (c0 + vc < values ? v[x] : 1.f) : 0.f);
        bf16 wh, wl;
        split_bf16(expf(f_last + j[x] - m_last) * (float)value, wh, wl);
        plain[x] = value, hi[x] = wh, lo[x] = wl;
      }
      *(run_t*)(v_t[0] + vc * VLD + vt0) = plain;
      *(run_t*)(v_t[1] + vc * VLD + vt0) = hi;
      *(run_t*)(v_t[2] + vc * VLD + vt0) = lo;
    }
#pragma unroll
    for (int b = 0; b < DB; ++b) {
      bf16x4 hi, lo;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        bf16 sh, sl;
        split_bf16(S[b][i], sh, sl);
        hi[i] = sh, lo[i] = sl;
      }
      const int at = c * SLD + (wave * DB + b) * 16 + g * 4;
      *(bf16x4*)(s_hi + at) = hi;
      *(bf16x4*)(s_lo + at) = lo;
    }
    __syncthreads();
    const float decay = expf(m + f_last - m_last);
    fetch_values(chunk + 1);
    // (the state's fragments two products' worth ahead, and a sum of its own for each half: no product waits for the LDS or for the
    // one before it)
    floatx4 past = {0.f, 0.f, 0.f, 0.f}, past_lo = past, here = past, here_lo = past;
    bf16x8 part[3][2];
    auto state_part = [&](int x) {
      part[x % 3][0] = *(const bf16x8*)(s_hi + c * SLD + x * 32 + g * 8);
      part[x % 3][1] = *(const bf16x8*)(s_lo + c * SLD + x * 32 + g * 8);
    };
    state_part(0);
    state_part(1);
    bf16x8 vf[3][2];
#pragma unroll
    for (int x = 0; x < QK; ++x) {
      if (x + 2 < QK) {
        state_part(x + 2);
      } else {
        const int y = x - (QK - 2);                        // the values' fragments behind the state's last
#pragma unroll
        for (int n = 0; n < 3; ++n) vf[n][y] = *(const bf16x8*)(v_t[n] + c * VLD + y * 32 + g * 8);
      }
      __builtin_amdgcn_sched_barrier(0);
      past = __builtin_amdgcn_mfma_f32_16x16x32_bf16(q[x], part[x % 3][0], past, 0, 0, 0);
      past_lo = __builtin_amdgcn_mfma_f32_16x16x32_bf16(q[x], part[x % 3][1], past_lo, 0, 0, 0);
      __builtin_amdgcn_sched_barrier(0);
    }
    fetch_q(chunk + 1);
#pragma unroll
    for (int b = 0; b < DB; ++b) S[b] *= decay;
    here = __builtin_amdgcn_mfma_f32_16x16x32_bf16(p[0][0], vf[0][0], here, 0, 0, 0);
    here_lo = __builtin_amdgcn_mfma_f32_16x16x32_bf16(p[1][0], vf[0][0], here_lo, 0, 0, 0);
    if (wave >= 2) {                                       // (tokens of the chunk's first half see nothing of its second)
      here = __builtin_amdgcn_mfma_f32_16x16x32_bf16(p[0][1], vf[0][1], here, 0, 0, 0);
      here_lo = __builtin_amdgcn_mfma_f32_16x16x32_bf16(p[1][1], vf[0][1], here_lo, 0, 0, 0);
    }
#pragma unroll
    for (int x = 0; x < 2; ++x)
#pragma unroll
      for (int half = 0; half < 2; ++half)
#pragma unroll
        for (int b = 0; b < DB; ++b) S[b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k[b][x], vf[1 + half][x], S[b], 0, 0, 0);
    fetch_p(chunk + 1);
    fetch_k(chunk + 1);
    const floatx4 from_state = *(const floatx4*)(of_state + wave * 16 + g * 4), from_chunk = *(const floatx4*)(of_chunk + wave * 16 + g * 4);
    float* row = raw + ((int64_t)(start + chunk * L + wave * 16 + g * 4) * H + h) * columns + c0 + c;
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (wave * 16 + g * 4 + i < count && c0 + c < columns)
        row[(int64_t)i * H * columns] = fmaf(from_state[i], past[i] + past_lo[i], from_chunk[i] * (here[i] + here_lo[i]));
    if (blockIdx.z == 0 && tid < count) floors[(int64_t)(start + chunk * L + tid) * H + h] = floor_here;
    m = m_last;
    __syncthreads();
  }

#pragma unroll
  for (int b = 0; b < DB; ++b) *(floatx4*)(s_f32 + c * FLD + (wave * DB + b) * 16 + g * 4) = S[b];
  __syncthreads();
  for (int e = tid; e < ROWS * C * SPLIT; e += THREADS) {
    const int row = e / (C * SPLIT), cc = e / SPLIT % C, s = e % SPLIT;
    if (c0 + cc < columns) st[((int64_t)row * columns + c0 + cc) * SPLIT + s] = s_f32[cc * FLD + s * ROWS + row];
  }
  if (tid == 0 && blockIdx.z == 0) maxima[(int64_t)r * H + h] = m;
}

}  // namespace

// Slots of the packs that a step of so many tokens and requests needs, and what a (slot, head) takes of each, in elements.
LRS_API int lrs_mlstm_slots(int tokens, int requests) { return tokens / L + requests + 1; }

// lrs_mlstm for steps with long portions in bfloat16 (out is bfloat16): the same arguments, with maxima [requests, H] float32 for its
// `gates`, and the packs: q_pack and k_pack bfloat16 [slots, H, 64 * (16 * state rows)], p_pack bfloat16 [slots, H, 2 * 64 * 64],
// gate_pack float32 [slots, H, 3 * 64], slots = lrs_mlstm_slots(tokens, requests).  singles: that many requests at the head of the step
// bring one token each (their tokens are its first); they go to the kernel for single tokens, which does not walk a chunk for one.
LRS_API int lrs_mlstm_chunks(void* out, const float* proj, int ld, int tokens, int requests, const int* token_request, const int* cu,
                             const int* slot_ids, float* state, int64_t state_stride, int H, int d, int dv, const float* i_bias,
                             const float* f_bias, float cap, const float* norm_w, float eps, float* maxima, float* floors, float* raw,
                             void* q_pack, void* k_pack, void* p_pack, float* gate_pack, int singles, void* stream) {
  LRS_REQUIRE(tokens > 0 && requests > 0 && requests <= tokens, "mlstm_chunks: bad sizes tokens=%d requests=%d", tokens, requests);
  LRS_REQUIRE(H > 0 && d > 0 && dv > 0 && d <= 256, "mlstm_chunks: bad sizes H=%d d=%d dv=%d (keys of up to 256 values)", H, d, dv);
  LRS_REQUIRE(singles >= 0 && singles < requests, "mlstm_chunks: %d single tokens leave no portion among %d requests", singles, requests);
  LRS_REQUIRE(cap > 0.f && eps > 0.f, "mlstm_chunks: the gates' cap and eps must be positive");
  const int rows = lrs_delta_state_rows(d), columns = dv + 1;
  const int k_at = H * d, v_at = 2 * H * d, g_at = v_at + H * dv, i_at = g_at + H * dv, f_at = i_at + H;
  LRS_REQUIRE(ld >= f_at + H, "mlstm_chunks: projection rows of %d hold fewer than the %d columns needed", ld, f_at + H);
  const int64_t m_offset = (int64_t)H * rows * SPLIT * columns;
  LRS_REQUIRE(state_stride >= m_offset + H, "mlstm_chunks: a state row of %lld floats is too short", (long long)state_stride);
  LRS_REQUIRE((((uintptr_t)proj | (uintptr_t)q_pack | (uintptr_t)k_pack | (uintptr_t)p_pack) % 16) == 0, "mlstm_chunks: rows and packs must be 16 bytes aligned");
  hipStream_t s = (hipStream_t)stream;
  // what follows sees the requests behind the single ones (token numbers stay those of the step)
  if (singles > 0)
    lrs_mlstm_singles(proj, ld, singles, slot_ids, state, state_stride, H, d, dv, i_bias, f_bias, cap, raw, floors, maxima, s);
  const int* rest_cu = cu + singles;
  const int* rest_slots = slot_ids + singles;
  float* rest_maxima = maxima + (int64_t)singles * H;
  const int rest = requests - singles;
  const dim3 pgrid(lrs_mlstm_slots(tokens, rest), H);
  // 32 columns a workgroup, or 16 where that leaves half of the chip idle
  const bool wide = (int64_t)rest * H * ((columns + 31) / 32) >= 96;
  const dim3 grid(rest, H, wide ? (columns + 31) / 32 : (columns + 15) / 16);
#define WALK(DP, CB)                                                                                                                        \
  mlstm_chunks_kernel<DP, CB><<<grid, 256 * CB, 0, s>>>(proj, ld, v_at, (const bf16*)q_pack, (const bf16*)k_pack, (const bf16*)p_pack, gate_pack, \
                                                   rest_cu, rest_slots, state, state_stride, m_offset, H, columns, raw, floors, rest_maxima)
#define RUN(DP)                                                                                                                        \
  do {                                                                                                                                 \
    mlstm_pack_kernel<DP><<<pgrid, 256, 0, s>>>(proj, ld, k_at, i_at, f_at, i_bias, f_bias, cap, rest_cu, rest, H, d, (bf16*)q_pack,     \
                                                (bf16*)k_pack, (bf16*)p_pack, gate_pack);                                              \
    if (wide) WALK(DP, 2);                                                                                                             \
    else WALK(DP, 1);                                                                                                                  \
  } while (0)
  if (rows == 4) RUN(64);
  else if (rows == 8) RUN(128);
  else RUN(256);
#undef RUN
#undef WALK
  if (lrs_check_launch("mlstm_chunks")) return 1;
  return lrs_mlstm_read_out(out, LRS_BF16, raw, floors, proj, ld, g_at, norm_w, 1.0f / sqrtf((float)d), eps, tokens, requests, H, dv, maxima,
                            token_request, cu, slot_ids, state, state_stride, m_offset, s);
}
