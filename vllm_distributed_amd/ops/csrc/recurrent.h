// Pieces shared by the linear-recurrence kernels (linear_attention.hip, delta_rule.hip).
//
// Chunk-parallel forms run on the fp32 matrix instruction v_mfma_f32_16x16x4_f32: operands and sums stay in 32 bits, so
// a prompt may be cut anywhere without anything but the order of fp32 sums changing.  Its register layout (lane l,
// g = l / 16):  A[i = l % 16][k = g],  B[k = g][j = l % 16],  C / D register r = [i = 4 g + r][j = l % 16].
// All products here take their K index in the order k = 4 g + r (step r, lane group g), so that
//   * an accumulator is, as it stands, the B operand of a next product over its rows, and
//   * an accumulator holding a transposed product is, as it stands, the A operand over its rows,
// and no result has to travel through LDS between chained products.
#pragma once
#include "common.h"

__device__ __forceinline__ f32x4 mfma_f32(float a, float b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}

// c += A B over 16 consecutive k: a[r], b[r] belong to k = 4 g + r
__device__ __forceinline__ f32x4 mfma_f32_k16(f32x4 a, f32x4 b, f32x4 c) {
#pragma unroll
  for (int r = 0; r < 4; ++r) c = mfma_f32(a[r], b[r], c);
  return c;
}

// two such products in turn: neither waits for the step right before it
__device__ __forceinline__ void mfma_f32_k16_two(f32x4 a0, f32x4 b0, f32x4& c0, f32x4 a1, f32x4 b1, f32x4& c1) {
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    c0 = mfma_f32(a0[r], b0[r], c0);
    c1 = mfma_f32(a1[r], b1[r], c1);
  }
}

// sum over the 16 lanes of a DPP row, result in every lane
__device__ __forceinline__ float row16_sum(float v) {
  v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0xB1, 0xF, 0xF, true));
  v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0x4E, 0xF, 0xF, true));
  v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0x141, 0xF, 0xF, true));
  v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0x140, 0xF, 0xF, true));
  return v;
}

__device__ __forceinline__ float rec_sigmoid(float v) { return 1.f / (1.f + expf(-v)); }
__device__ __forceinline__ float rec_softplus(float v) { return v > 20.f ? v : log1pf(expf(v)); }
__device__ __forceinline__ float rec_logsigmoid(float v) { return fminf(v, 0.f) - log1pf(expf(-fabsf(v))); }

// four consecutive values p[0 .. 3], those from n on as zeros; vec: p is aligned for a 4-value load
template <typename T> __device__ __forceinline__ f32x4 load4(const T* p, int n, bool vec) {
  f32x4 o = {0.f, 0.f, 0.f, 0.f};
  if (n <= 0) return o;
  if (vec && n >= 4) {
    const typename Vec<T>::v4 v = *reinterpret_cast<const typename Vec<T>::v4*>(p);
#pragma unroll
    for (int i = 0; i < 4; ++i) o[i] = (float)v[i];
  } else {
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (i < n) o[i] = (float)p[i];
  }
  return o;
}

__device__ __forceinline__ void store4(float* p, f32x4 v, int n, bool vec) {
  if (n <= 0) return;
  if (vec && n >= 4) {
    *reinterpret_cast<f32x4*>(p) = v;
  } else {
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (i < n) p[i] = v[i];
  }
}

// One-token form: a column's D state values are spread over sixteen neighbouring lanes, NR per lane.  Lane `part` holds
// the values d(i), i < NR: groups of four consecutive values, 64 apart (NR >= 4), so a column is read and written as
// whole 256-byte runs.
template <int NR> __device__ __forceinline__ int rec_lane_value(int part, int i) {
  return NR >= 4 ? (i / 4 * 16 + part) * 4 + i % 4 : part * NR + i;
}

template <int NR> __device__ __forceinline__ void rec_load_column(float* S, const float* col, int part, int D, bool live,
                                                                  bool vec) {
  if constexpr (NR >= 4) {
#pragma unroll
    for (int i = 0; i < NR; i += 4) {
      const int d = rec_lane_value<NR>(part, i);
      const f32x4 v = load4<float>(col + d, live ? D - d : 0, vec);
      S[i] = v[0]; S[i + 1] = v[1]; S[i + 2] = v[2]; S[i + 3] = v[3];
    }
  } else {
#pragma unroll
    for (int i = 0; i < NR; ++i) {
      const int d = rec_lane_value<NR>(part, i);
      S[i] = live && d < D ? col[d] : 0.f;
    }
  }
}

template <int NR> __device__ __forceinline__ void rec_store_column(const float* S, float* col, int part, int D, bool vec) {
  if constexpr (NR >= 4) {
#pragma unroll
    for (int i = 0; i < NR; i += 4) {
      const int d = rec_lane_value<NR>(part, i);
      store4(col + d, f32x4{S[i], S[i + 1], S[i + 2], S[i + 3]}, D - d, vec);
    }
  } else {
#pragma unroll
    for (int i = 0; i < NR; ++i) {
      const int d = rec_lane_value<NR>(part, i);
      if (d < D) col[d] = S[i];
    }
  }
}

// the lane's NR values of an LDS row (rows hold 16 * NR values, zeros beyond D)
template <int NR> __device__ __forceinline__ void rec_lane_row(float* o, const float* row, int part) {
  if constexpr (NR >= 4) {
#pragma unroll
    for (int i = 0; i < NR; i += 4) {
      const f32x4 v = *reinterpret_cast<const f32x4*>(row + rec_lane_value<NR>(part, i));
      o[i] = v[0]; o[i + 1] = v[1]; o[i + 2] = v[2]; o[i + 3] = v[3];
    }
  } else {
#pragma unroll
    for (int i = 0; i < NR; ++i) o[i] = row[rec_lane_value<NR>(part, i)];
  }
}

// out[t, h, :] = o / sqrt(mean(o^2) + eps) * norm_w * silu(gate) over a head's Dv values, for the tokens of sequences
// seq0 + blockIdx.y with more than `limit` new tokens: one wave per (token, head).  norm_w may be null (no weight); its
// rows of Dv values lie norm_head apart (0: one row for all heads).
template <typename T>
__global__ __launch_bounds__(256) void head_norm_silu_kernel(T* __restrict__ out, long o_stride,
                                                             const float* __restrict__ o_raw,
                                                             const T* __restrict__ gate, long g_stride,
                                                             const float* __restrict__ norm_w, int norm_head,
                                                             const int* __restrict__ qsl,
                                                             const int* __restrict__ seq_lens, int seq0, int limit,
                                                             int H, int Dv, float eps) {
  const int s = seq0 + blockIdx.y;
  if (seq_lens[s] <= 0) return;
  const int t0 = qsl[s], L = qsl[s + 1] - t0;
  const long row = (long)blockIdx.x * 4 + (threadIdx.x >> 6);             // (token of the sequence, head)
  if (L <= limit || row >= (long)L * H) return;
  const int lane = threadIdx.x & 63;
  const long t = t0 + row / H;
  const int h = (int)(row % H);
  const float* o = o_raw + (t * H + h) * (long)Dv;
  float ss = 0.f;
  for (int j = lane; j < Dv; j += 64) ss += o[j] * o[j];
  ss = wave_sum(ss);
  const float rs = 1.f / sqrtf(ss / (float)Dv + eps);
  for (int j = lane; j < Dv; j += 64) {
    const float z = (float)gate[t * g_stride + (long)h * Dv + j];
    out[t * o_stride + (long)h * Dv + j] = (T)(o[j] * rs * (norm_w ? norm_w[(long)h * norm_head + j] : 1.f) * z * rec_sigmoid(z));
  }
}
