// Token shift of RWKV-style mixers over a ragged batch: every one of M mixes of a token reads
//     h + (h' - h) * mu[m]                      h': the row of the token before it in the same sequence
// The row before a portion's first token is the one its state slot holds (zeros when the sequence starts in this step);
// the portion's last row replaces it.  A thread owns VEC columns of a run of consecutive tokens, reads every row once and
// writes all mixes; the run that holds a sequence's first token reads its slot and then stores the last row into it, so
// that no other thread touches those columns of the slot.
#include "common.h"

constexpr int SHIFT_RUN = 8;                   // tokens per thread

template <typename T, int VEC>
__global__ __launch_bounds__(256) void token_shift_mix_kernel(T* __restrict__ out, long out_mix, const T* __restrict__ h,
                                                              long h_stride, const float* __restrict__ mu,
                                                              T* __restrict__ state, const int* __restrict__ qsl,
                                                              const int* __restrict__ seq_lens,
                                                              const int* __restrict__ slot_table, long st_stride, int M,
                                                              int W) {
  using V = T __attribute__((ext_vector_type(VEC)));
  const int s = blockIdx.y, c = (blockIdx.z * 256 + threadIdx.x) * VEC;
  const int sl = seq_lens[s];
  if (sl <= 0 || c >= W) return;
  const int t0 = qsl[s], L = qsl[s + 1] - t0, first = blockIdx.x * SHIFT_RUN;
  if (first >= L) return;
  const int n = min(SHIFT_RUN, L - first);
  const T* hp = h + (long)(t0 + first) * h_stride + c;
  V x[SHIFT_RUN], before;
#pragma unroll
  for (int i = 0; i < SHIFT_RUN; ++i)
    if (i < n) x[i] = *reinterpret_cast<const V*>(hp + i * h_stride);
  if (first > 0) {
    before = *reinterpret_cast<const V*>(hp - h_stride);
  } else {
    T* row = state + (long)slot_table[s * st_stride] * W + c;
    if (sl - L > 0) {
      before = *reinterpret_cast<const V*>(row);
    } else {
#pragma unroll
      for (int j = 0; j < VEC; ++j) before[j] = (T)0.f;
    }
    *reinterpret_cast<V*>(row) = *reinterpret_cast<const V*>(hp + (long)(L - 1) * h_stride);
  }
  for (int m = 0; m < M; ++m) {
    float f[VEC];
#pragma unroll
    for (int j = 0; j < VEC; ++j) f[j] = mu[(long)m * W + c + j];
    T* op = out + m * out_mix + (long)(t0 + first) * W + c;
    V p = before;
#pragma unroll
    for (int i = 0; i < SHIFT_RUN; ++i)
      if (i < n) {
        V o;
#pragma unroll
        for (int j = 0; j < VEC; ++j) {
          const float v = (float)x[i][j];
          o[j] = (T)(v + ((float)p[j] - v) * f[j]);
        }
        *reinterpret_cast<V*>(op + (long)i * W) = o;
        p = x[i];
      }
  }
}

VDA_EXPORT int vda_token_shift_mix(void* out, long out_mix, const void* h, long h_stride, const float* mu, void* state,
                                   const int* qsl, const int* seq_lens, const int* slot_table, long st_stride, int T, int S,
                                   int M, int W, int max_q, int dtype, hipStream_t st) {
  if (T <= 0 || S <= 0) return 0;
  if (W < 1 || M < 1 || max_q < 1) return -1;
  const int V = W % 4 == 0 && h_stride % 4 == 0 && out_mix % 4 == 0 && (uintptr_t)h % 16 == 0 && (uintptr_t)out % 16 == 0 &&
                        (uintptr_t)state % 16 == 0
                    ? 4
                    : 1;
  const dim3 grid((max_q + SHIFT_RUN - 1) / SHIFT_RUN, S, (W / V + 255) / 256);
#define L2(TT, VV) hipLaunchKernelGGL((token_shift_mix_kernel<TT, VV>), grid, dim3(256), 0, st, (TT*)out, out_mix,     \
                                      (const TT*)h, h_stride, mu, (TT*)state, qsl, seq_lens, slot_table, st_stride, M, W)
#define L(TT) do { if (V == 4) L2(TT, 4); else L2(TT, 1); } while (0)
  if (dtype == VDA_BF16) L(bf16_t);
  else if (dtype == VDA_F16) L(f16_t);
  else if (dtype == VDA_F32) L(float);
  else return -3;
#undef L
#undef L2
  VDA_CHECK_LAUNCH();
  return 0;
}
