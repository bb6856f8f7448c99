// Gated delta rule with one decay per head and key channel, over a ragged batch with per-request state slots.
//
// Per head, with S a [D, Dv] matrix kept in fp32 (stored transposed, [Dv, D], so that a column is contiguous):
//     S <- diag(decay) S;   u = beta (v - S^T k);   S <- S + k u^T;   o = S^T q
// where q and k are unit vectors (q also times D^-1/2), decay = exp(-exp(a_log) * softplus(a + dt_bias)) and
// beta = sigmoid(b).  The read-out sees the token's own write.  The output is RMS-normalised over Dv, scaled by a
// weight shared by the heads and gated by sigmoid(gate).
//
// Two kernels and a small epilogue:
//   prepare  (parallel over tokens)  unit vectors q^, k^ per q/k head, decays per head and key channel, beta and
//            q^ . k^ per head, all fp32, rows padded with zeros to a multiple of 16 channels;
//   scan     every column of S evolves on its own given (q^, k^, decay, beta), so a workgroup owns one (sequence,
//            head, 16 columns) and sixteen adjacent lanes share a column, NR = D/16 rows each in registers.  The two
//            dot products of a step (k^ . dS and q^ . dS on the decayed state, o = q^ . dS + (q^ . k^) u) are summed
//            over the sixteen lanes with DPP row operations.  The prepared vectors of 32 tokens sit in LDS while
//            the next 32 are on their way from memory, so a step is one short dependent chain of register work.
//   epilogue normalises the read-out over the head's columns, applies the weight and the gate.
// With ONE decay per head (vda_gated_delta_rule_head: g = exp(-exp(a_log) softplus(a + dt_bias)), gate silu) two other
// kernels do the work:
//   step     sequences with at most 16 new tokens: one workgroup per (sequence, head) does everything -- unit vectors,
//            gates, the recurrence token by token with the state read and written once, output norm and gate;
//   chunked  longer ones, sixteen tokens at a time on the fp32 matrix instruction.  With b the running sum of log g,
//            M_ij = beta_i e^(b_i - b_j) k_i.k_j (j < i) and T = (I + M)^-1 diag(beta), a block's writes are
//                U = T (V - diag(e^b) K S),   O = diag(e^b) Q S + P U,   P_ij = e^(b_i - b_j) q_i.k_j (j <= i)
//                S <- e^b_n S + K^T diag(e^(b_n - b)) U
//            T, P and the unit vectors of every block are made in parallel (delta_block_prepare); the walk over the blocks
//            keeps S of sixteen columns in a wave's accumulators and passes every product on in registers
//            (recurrent.h); norm and gate follow in a launch of their own.
// The batch description is the one of the other recurrent kernels (qsl, seq_lens, slot in column 0 of the table;
// a sequence carries state in when seq_len - new_tokens > 0), so prompts, portions of prompts, single decoded
// tokens and mixtures of them are one code path, and the state after a token does not depend on how the
// sequence was cut.
#include "recurrent.h"

// grid: tokens; one wave per (token, vector): G query vectors, G key vectors (with their dot products), H decays
template <typename T>
__global__ __launch_bounds__(256) void delta_prepare_kernel(
    float* __restrict__ qhat, float* __restrict__ khat, float* __restrict__ dec, float* __restrict__ sc,
    const T* __restrict__ qkv, long qkv_stride, const T* __restrict__ a_raw, long a_stride,
    const T* __restrict__ b_raw, long b_stride, const float* __restrict__ a_log, const float* __restrict__ dt_bias,
    int H, int G, int D, int Dp) {
  const long t = blockIdx.x;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const float q_scale = 1.f / sqrtf((float)D);
  const int rep = H / G;
  for (int v = wave; v < G + H; v += 4) {
    if (v < G) {
      const T* qr = qkv + t * qkv_stride + (long)v * D;
      const T* kr = qkv + t * qkv_stride + (long)(G + v) * D;
      float sq = 0.f, sk = 0.f;
      for (int d = lane; d < D; d += 64) {
        const float a = (float)qr[d], b = (float)kr[d];
        sq += a * a;
        sk += b * b;
      }
      sq = wave_sum(sq);
      sk = wave_sum(sk);
      const float rq = q_scale / sqrtf(sq + 1e-6f), rk = 1.f / sqrtf(sk + 1e-6f);
      float dot = 0.f;
      for (int d = lane; d < Dp; d += 64) {
        const float a = d < D ? (float)qr[d] * rq : 0.f, b = d < D ? (float)kr[d] * rk : 0.f;
        qhat[(t * G + v) * Dp + d] = a;
        khat[(t * G + v) * Dp + d] = b;
        dot += a * b;
      }
      dot = wave_sum(dot);
      // per head: [beta, q^ . k^]
      for (int h = v * rep + lane; h < (v + 1) * rep; h += 64) {
        sc[(t * H + h) * 2] = rec_sigmoid((float)b_raw[t * b_stride + h]);
        sc[(t * H + h) * 2 + 1] = dot;
      }
    } else {
      const int h = v - G;
      const float a_scale = expf(a_log[h]);
      for (int d = lane; d < Dp; d += 64)
        dec[(t * H + h) * Dp + d] =
            d < D ? expf(-a_scale * rec_softplus((float)a_raw[t * a_stride + (long)h * D + d] + dt_bias[(long)h * D + d]))
                  : 0.f;
    }
  }
}


// grid (heads, sequences, groups of 16 columns); block 256 = 16 columns x 16 lanes.  The prepared vectors of 32
// tokens are staged in LDS; the next 32 are on their way from memory (into registers) while these are computed.
template <typename T, int NR>
__global__ __launch_bounds__(256) void gated_delta_rule_kernel(
    float* __restrict__ o_raw, const T* __restrict__ qkv, long qkv_stride, const float* __restrict__ qhat,
    const float* __restrict__ khat, const float* __restrict__ dec, const float* __restrict__ sc,
    float* __restrict__ state, const int* __restrict__ qsl, const int* __restrict__ seq_lens,
    const int* __restrict__ slot_table, long st_stride, int H, int G, int D, int Dv) {
  constexpr int Dp = 16 * NR;
  constexpr int DR_CT = NR >= 16 ? 16 : 32;            // tokens staged in LDS at a time (48 KiB at most)
  constexpr int NV = DR_CT * 16 / 256;                 // value elements a thread carries per chunk
  constexpr int VPT = DR_CT * Dp / 4;                  // float4 per staged vector kind
  constexpr int PF = (3 * VPT + 255) / 256;            // float4 a thread carries per chunk
  __shared__ __align__(16) float kqg[3 * DR_CT * Dp];  // k^ | q^ | decay, [kind][token][Dp]
  __shared__ float vv[DR_CT * 16];
  __shared__ float sc2[DR_CT * 2];
  const int h = blockIdx.x, s = blockIdx.y, tid = threadIdx.x;
  const int sl = seq_lens[s];
  if (sl <= 0) return;
  const int t0 = qsl[s], L = qsl[s + 1] - t0;
  if (L <= 0) return;
  const int c = h / (H / G);
  const int col0 = blockIdx.z * 16;
  const int col = col0 + (tid >> 4), part = tid & 15;
  const bool has_col = col < Dv;
  float* Scol = state + (((long)slot_table[s * st_stride] * H + h) * Dv + (has_col ? col : Dv - 1)) * D + part * NR;
  float S[NR];
  const bool carry = sl - L > 0;
#pragma unroll
  for (int i = 0; i < NR; ++i) S[i] = (carry && part * NR + i < D) ? Scol[i] : 0.f;

  f32x4 pre[PF];
  float pv[NV], ps = 0.f;
  auto prefetch = [&](int cs) {
    const int nt = min(DR_CT, L - cs);
#pragma unroll
    for (int n = 0; n < PF; ++n) {
      const int e = tid + n * 256;
      f32x4 x = {0.f, 0.f, 0.f, 0.f};
      if (e < 3 * VPT) {
        const int kind = e / VPT, rem = e - kind * VPT, tt = rem / (Dp / 4), j = rem - tt * (Dp / 4);
        if (tt < nt) {
          const long t = t0 + cs + tt;
          const float* src = kind == 0 ? khat + (t * G + c) * Dp : kind == 1 ? qhat + (t * G + c) * Dp
                                                                             : dec + (t * H + h) * Dp;
          x = *reinterpret_cast<const f32x4*>(src + 4 * j);
        }
      }
      pre[n] = x;
    }
#pragma unroll
    for (int n = 0; n < NV; ++n) {
      const int e = tid + n * 256, tt = e >> 4, j = e & 15;
      pv[n] = (tt < nt && col0 + j < Dv)
                  ? (float)qkv[(long)(t0 + cs + tt) * qkv_stride + (long)2 * G * D + (long)h * Dv + col0 + j] : 0.f;
    }
    if (tid < 2 * DR_CT) ps = (tid >> 1) < nt ? sc[((long)(t0 + cs + (tid >> 1)) * H + h) * 2 + (tid & 1)] : 0.f;
  };

  prefetch(0);
  for (int cs = 0; cs < L; cs += DR_CT) {
    const int nt = min(DR_CT, L - cs);
    __syncthreads();                                   // the previous chunk has been read by everybody
#pragma unroll
    for (int n = 0; n < PF; ++n) {
      const int e = tid + n * 256;
      if (e < 3 * VPT) *reinterpret_cast<f32x4*>(kqg + 4 * e) = pre[n];
    }
#pragma unroll
    for (int n = 0; n < NV; ++n) vv[tid + n * 256] = pv[n];
    if (tid < 2 * DR_CT) sc2[tid] = ps;
    __syncthreads();
    if (cs + DR_CT < L) prefetch(cs + DR_CT);
    for (int tt = 0; tt < nt; ++tt) {
      const float* kp = kqg + tt * Dp + part * NR;
      const float* qp = kp + DR_CT * Dp;
      const float* gp = qp + DR_CT * Dp;
      float kr[NR], r = 0.f, p = 0.f;
      if constexpr (NR >= 4) {
#pragma unroll
        for (int i = 0; i < NR / 4; ++i) {
          const f32x4 k4 = reinterpret_cast<const f32x4*>(kp)[i], q4 = reinterpret_cast<const f32x4*>(qp)[i],
                      g4 = reinterpret_cast<const f32x4*>(gp)[i];
#pragma unroll
          for (int j = 0; j < 4; ++j) {
            const float sd = S[4 * i + j] * g4[j];
            S[4 * i + j] = sd;
            kr[4 * i + j] = k4[j];
            r += sd * k4[j];
            p += sd * q4[j];
          }
        }
      } else {
#pragma unroll
        for (int i = 0; i < NR; ++i) {
          const float sd = S[i] * gp[i];
          S[i] = sd;
          kr[i] = kp[i];
          r += sd * kp[i];
          p += sd * qp[i];
        }
      }
      r = row16_sum(r);
      p = row16_sum(p);
      const float u = sc2[2 * tt] * (vv[tt * 16 + (tid >> 4)] - r);
#pragma unroll
      for (int i = 0; i < NR; ++i) S[i] += kr[i] * u;
      if (part == 0 && has_col) o_raw[(long)(t0 + cs + tt) * H * Dv + (long)h * Dv + col] = p + sc2[2 * tt + 1] * u;
    }
  }
  if (has_col) {
#pragma unroll
    for (int i = 0; i < NR; ++i)
      if (part * NR + i < D) Scol[i] = S[i];
  }
}

// out[t, h, :] = o / sqrt(mean(o^2) + eps) * norm_w * sigmoid(gate): one wave per (token, head)
template <typename T>
__global__ __launch_bounds__(256) void delta_out_norm_gate_kernel(T* __restrict__ out, long o_stride,
                                                                  const float* __restrict__ o_raw,
                                                                  const T* __restrict__ gate_raw, long g_stride,
                                                                  const float* __restrict__ norm_w, long rows, int H,
                                                                  int Dv, float eps) {
  const long row = (long)blockIdx.x * 4 + (threadIdx.x >> 6);      // (token, head) pair
  if (row >= rows) return;
  const int lane = threadIdx.x & 63;
  const long t = row / H;
  const int h = (int)(row % H);
  const float* o = o_raw + row * Dv;
  float ss = 0.f;
  for (int j = lane; j < Dv; j += 64) ss += o[j] * o[j];
  ss = wave_sum(ss);
  const float rs = 1.f / sqrtf(ss / (float)Dv + eps);
  for (int j = lane; j < Dv; j += 64) {
    const float gt = rec_sigmoid((float)gate_raw[t * g_stride + (long)h * Dv + j]);
    out[t * o_stride + (long)h * Dv + j] = (T)(o[j] * rs * norm_w[j] * gt);
  }
}

template <typename T>
static int launch_delta_rule(int NR, dim3 grid, hipStream_t st, float* o_raw, const void* qkv, long qkv_stride,
                             const float* qhat, const float* khat, const float* dec, const float* sc, float* state,
                             const int* qsl, const int* seq_lens, const int* slot_table, long st_stride, int H, int G,
                             int D, int Dv) {
#define L(NRV)                                                                                                     \
  hipLaunchKernelGGL((gated_delta_rule_kernel<T, NRV>), grid, dim3(256), 0, st, o_raw, (const T*)qkv, qkv_stride,  \
                     qhat, khat, dec, sc, state, qsl, seq_lens, slot_table, st_stride, H, G, D, Dv)
  switch (NR) {
    case 1: L(1); break;
    case 2: L(2); break;
    case 4: L(4); break;
    case 8: L(8); break;
    case 16: L(16); break;
    default: return -2;
  }
#undef L
  return 0;
}

// channels per lane of the scan for key width D (D <= 256), and the padded row length of the prepared vectors
VDA_EXPORT int vda_delta_rule_padded_dim(int D) {
  int NR = 1;
  while (16 * NR < D) NR *= 2;
  return 16 * NR;
}

// o_raw: fp32 [T, H * Dv]; prep: fp32 scratch of T * ((2 G + H) * Dp + 2 H) floats, Dp = vda_delta_rule_padded_dim(D)
VDA_EXPORT int vda_gated_delta_rule(void* out, long o_stride, float* o_raw, float* prep, const void* qkv,
                                    long qkv_stride, const void* a_raw, long a_stride, const void* b_raw,
                                    long b_stride, const void* gate_raw, long g_stride, const float* a_log,
                                    const float* dt_bias, const float* norm_w, float* state, const int* qsl,
                                    const int* seq_lens, const int* slot_table, long st_stride, int T_tokens, int S,
                                    int H, int G, int D, int Dv, float eps, int dtype, hipStream_t st) {
  if (S <= 0 || T_tokens <= 0) return 0;
  if (H <= 0 || G <= 0 || H % G || D < 1 || D > 256 || Dv < 1) return -1;
  const int Dp = vda_delta_rule_padded_dim(D), NR = Dp / 16;
  float* qhat = prep;
  float* khat = qhat + (size_t)T_tokens * G * Dp;
  float* dec = khat + (size_t)T_tokens * G * Dp;
  float* sc = dec + (size_t)T_tokens * H * Dp;
#define LP(TT) hipLaunchKernelGGL((delta_prepare_kernel<TT>), dim3(T_tokens), dim3(256), 0, st, qhat, khat, dec, sc, \
                                  (const TT*)qkv, qkv_stride, (const TT*)a_raw, a_stride, (const TT*)b_raw, b_stride, \
                                  a_log, dt_bias, H, G, D, Dp)
  if (dtype == VDA_BF16) LP(bf16_t);
  else if (dtype == VDA_F16) LP(f16_t);
  else if (dtype == VDA_F32) LP(float);
  else return -3;
#undef LP
  VDA_CHECK_LAUNCH();
  dim3 grid(H, S, (Dv + 15) / 16);
  int rc;
  if (dtype == VDA_BF16)
    rc = launch_delta_rule<bf16_t>(NR, grid, st, o_raw, qkv, qkv_stride, qhat, khat, dec, sc, state, qsl, seq_lens,
                                   slot_table, st_stride, H, G, D, Dv);
  else if (dtype == VDA_F16)
    rc = launch_delta_rule<f16_t>(NR, grid, st, o_raw, qkv, qkv_stride, qhat, khat, dec, sc, state, qsl, seq_lens,
                                  slot_table, st_stride, H, G, D, Dv);
  else
    rc = launch_delta_rule<float>(NR, grid, st, o_raw, qkv, qkv_stride, qhat, khat, dec, sc, state, qsl, seq_lens,
                                  slot_table, st_stride, H, G, D, Dv);
  if (rc) return rc;
  VDA_CHECK_LAUNCH();
  const long rows = (long)T_tokens * H;
  dim3 g2((unsigned)((rows + 3) / 4)), b2(256);
#define L2(TT) hipLaunchKernelGGL((delta_out_norm_gate_kernel<TT>), g2, b2, 0, st, (TT*)out, o_stride, o_raw, \
                                  (const TT*)gate_raw, g_stride, norm_w, rows, H, Dv, eps)
  if (dtype == VDA_BF16) L2(bf16_t);
  else if (dtype == VDA_F16) L2(f16_t);
  else L2(float);
#undef L2
  VDA_CHECK_LAUNCH();
  return 0;
}

// ---- one decay per head --------------------------------------------------------------------------------------------
struct DeltaHeadArgs {
  const void* qkv;              // [T, 2 G D + H Dv] convolved q | k | v
  long qkv_stride;
  const void *a_raw, *b_raw, *gate;
  long a_stride, b_stride, g_stride;
  const float *a_log, *dt_bias, *norm_w;
  float eps;
  float* state;                 // [slots, H, Dv, D]
  void* out;
  long o_stride;
  float* o_raw;                 // [T, H * Dv]
  const int *qsl, *seq_lens, *slot_table;
  long st_stride;
  int H, G, D, Dv, seq0, limit;
  // what the walk reads, every matrix in the order its operand registers are filled ([lane][4], see recurrent.h):
  float* vecs;                  // [blocks, G, 3, DT, 256]: unit keys, unit queries (token = lane % 16), keys with rows and
                                //   columns exchanged (channel = lane % 16)
  float* mats;                  // [blocks, H, DELTA_MAT]: T, P (256 each), e^b (16), e^(b_n - b) (16)
};
#define DELTA_MAT 544

// grid (H, S); columns over groups of sixteen lanes as in lin_step_kernel
template <typename T, int NR>
__global__ __launch_bounds__(256) void delta_step_kernel(const DeltaHeadArgs a, const int tile) {
  constexpr int NCG = NR <= 8 ? 4 : NR <= 16 ? 2 : 1;
  constexpr int DP = 16 * NR;
  extern __shared__ __align__(16) float lds[];
  const int h = blockIdx.x, s = blockIdx.y, tid = threadIdx.x;
  const int sl = a.seq_lens[s];
  if (sl <= 0) return;
  const int t0 = a.qsl[s], L = a.qsl[s + 1] - t0;
  if (L <= 0 || L > a.limit) return;
  const int D = a.D, Dv = a.Dv, G = a.G, c = h / (a.H / G);
  float* qs = lds;                                     // [tile][DP] unit vectors
  float* ks = qs + tile * DP;
  float* vs = ks + tile * DP;                          // [tile][Dv]
  float* os = vs + tile * Dv;                          // [tile][Dv]
  float* sc = os + tile * Dv;                          // [tile][4]: decay, beta, q^ . k^
  const int part = tid & 15, sub = tid >> 4, lane = tid & 63, wave = tid >> 6;
  const bool carry = sl - L > 0;
  const bool vs4 = (D & 3) == 0;
  float* Sb = a.state + ((long)a.slot_table[s * a.st_stride] * a.H + h) * (long)Dv * D;
  const float q_scale = 1.f / sqrtf((float)D), a_scale = expf(a.a_log[h]), dtb = a.dt_bias[h];
  const T* qkv = (const T*)a.qkv;
  float S[NCG][NR];
  auto load_group = [&](int c0, bool live) {
#pragma unroll
    for (int n = 0; n < NCG; ++n) {
      const int col = c0 + n * 16 + sub;
      rec_load_column<NR>(S[n], Sb + (long)(col < Dv ? col : Dv - 1) * D, part, D, live && col < Dv, vs4);
    }
  };
  load_group(0, carry);
  for (int b = 0; b < L; b += tile) {
    const int nt = min(tile, L - b);
    if (b > 0) { __syncthreads(); load_group(0, true); }
    for (int tt = wave; tt < nt; tt += 4) {            // one wave per token: unit vectors and scalars
      const long t = t0 + b + tt;
      const T* qr = qkv + t * a.qkv_stride + (long)c * D;
      const T* kr = qkv + t * a.qkv_stride + (long)(G + c) * D;
      float sq = 0.f, sk = 0.f, dot = 0.f;
      for (int d = lane; d < D; d += 64) {
        const float x = (float)qr[d], y = (float)kr[d];
        sq += x * x;
        sk += y * y;
        dot += x * y;
      }
      sq = wave_sum(sq);
      sk = wave_sum(sk);
      dot = wave_sum(dot);
      const float rq = q_scale / sqrtf(sq + 1e-6f), rk = 1.f / sqrtf(sk + 1e-6f);
      for (int d = lane; d < DP; d += 64) {
        qs[tt * DP + d] = d < D ? (float)qr[d] * rq : 0.f;
        ks[tt * DP + d] = d < D ? (float)kr[d] * rk : 0.f;
      }
      if (lane == 0) {
        sc[tt * 4] = expf(-a_scale * rec_softplus((float)((const T*)a.a_raw)[t * a.a_stride + h] + dtb));
        sc[tt * 4 + 1] = rec_sigmoid((float)((const T*)a.b_raw)[t * a.b_stride + h]);
        sc[tt * 4 + 2] = dot * rq * rk;
      }
    }
    for (int e = tid; e < nt * Dv; e += 256) {
      const int tt = e / Dv, cc = e - tt * Dv;
      vs[e] = (float)qkv[(long)(t0 + b + tt) * a.qkv_stride + (long)2 * G * D + (long)h * Dv + cc];
    }
    __syncthreads();
    for (int c0 = 0; c0 < Dv; c0 += 16 * NCG) {
      for (int tt = 0; tt < nt; ++tt) {
        float kr[NR], qr[NR];
        rec_lane_row<NR>(kr, ks + tt * DP, part);
        rec_lane_row<NR>(qr, qs + tt * DP, part);
        const float g = sc[tt * 4], beta = sc[tt * 4 + 1], qk = sc[tt * 4 + 2];
#pragma unroll
        for (int n = 0; n < NCG; ++n) {
          const int col = c0 + n * 16 + sub;
          float r = 0.f, p = 0.f;
#pragma unroll
          for (int i = 0; i < NR; ++i) {
            S[n][i] *= g;
            r += S[n][i] * kr[i];
            p += S[n][i] * qr[i];
          }
          r = row16_sum(r);
          p = row16_sum(p);
          const float u = beta * (vs[tt * Dv + (col < Dv ? col : Dv - 1)] - r);
#pragma unroll
          for (int i = 0; i < NR; ++i) S[n][i] += kr[i] * u;
          if (part == 0 && col < Dv) os[tt * Dv + col] = p + qk * u;
        }
      }
#pragma unroll
      for (int n = 0; n < NCG; ++n) {
        const int col = c0 + n * 16 + sub;
        if (col < Dv) rec_store_column<NR>(S[n], Sb + (long)col * D, part, D, vs4);
      }
      if (c0 + 16 * NCG < Dv) load_group(c0 + 16 * NCG, carry || b > 0);
    }
    __syncthreads();
    for (int tt = wave; tt < nt; tt += 4) {
      const long t = t0 + b + tt;
      const float* o = os + tt * Dv;
      float ss = 0.f;
      for (int cc = lane; cc < Dv; cc += 64) ss += o[cc] * o[cc];
      ss = wave_sum(ss);
      const float rs = 1.f / sqrtf(ss / (float)Dv + a.eps);
      for (int cc = lane; cc < Dv; cc += 64) {
        const float zg = (float)((const T*)a.gate)[t * a.g_stride + (long)h * Dv + cc];
        ((T*)a.out)[t * a.o_stride + (long)h * Dv + cc] = (T)(o[cc] * rs * a.norm_w[cc] * zg * rec_sigmoid(zg));
      }
    }
  }
}

// Blocks of sixteen tokens counted from every sequence's first new token; block index t0 / 16 + (s - seq0) + block.
// grid (blocks of the longest sequence, sequences, G): unit vectors of the block's q / k head, then, per value head that
// reads it, the block's matrices.
template <typename T, int DT>
__global__ __launch_bounds__(256) void delta_block_prepare_kernel(const DeltaHeadArgs a) {
  constexpr int DP = DT * 16, QP = DP + 4;
  __shared__ __align__(16) float qs[16 * QP], ks[16 * QP];
  __shared__ float M[4][16 * 17];
  const int srel = blockIdx.y, s = a.seq0 + srel, tid = threadIdx.x;
  if (a.seq_lens[s] <= 0) return;
  const int t0 = a.qsl[s], L = a.qsl[s + 1] - t0, tb = blockIdx.x * 16;
  if (L <= a.limit || tb >= L) return;
  const int n = min(16, L - tb), D = a.D, G = a.G, c = blockIdx.z;
  const int lane = tid & 63, wave = tid >> 6, lo = lane & 15, g = lane >> 4;
  const long blk = (long)(t0 / 16) + srel + blockIdx.x;
  const float q_scale = 1.f / sqrtf((float)D);
  float* vec = a.vecs + (blk * G + c) * 3 * 16 * DP;
  for (int tt = wave; tt < 16; tt += 4) {
    const T* qr = (const T*)a.qkv + (long)(t0 + tb + tt) * a.qkv_stride + (long)c * D;
    const T* kr = qr + (long)G * D;
    float sq = 0.f, sk = 0.f;
    if (tt < n)
      for (int d = lane; d < D; d += 64) {
        const float x = (float)qr[d], y = (float)kr[d];
        sq += x * x;
        sk += y * y;
      }
    sq = wave_sum(sq);
    sk = wave_sum(sk);
    const float rq = q_scale / sqrtf(sq + 1e-6f), rk = 1.f / sqrtf(sk + 1e-6f);
    for (int d = lane; d < DP; d += 64) {
      const bool ok = tt < n && d < D;
      const float x = ok ? (float)qr[d] * rq : 0.f, y = ok ? (float)kr[d] * rk : 0.f;
      qs[tt * QP + d] = x;
      ks[tt * QP + d] = y;
    }
  }
  __syncthreads();
  for (int e = tid; e < DT * 64; e += 256) {
    const int dt = e >> 6, tok = e & 15, g4 = (e >> 4 & 3) * 4;
    *reinterpret_cast<f32x4*>(vec + e * 4) = *reinterpret_cast<const f32x4*>(ks + tok * QP + dt * 16 + g4);
    *reinterpret_cast<f32x4*>(vec + 16 * DP + e * 4) = *reinterpret_cast<const f32x4*>(qs + tok * QP + dt * 16 + g4);
    const float* kc = ks + g4 * QP + dt * 16 + tok;
    *reinterpret_cast<f32x4*>(vec + 32 * DP + e * 4) = f32x4{kc[0], kc[QP], kc[2 * QP], kc[3 * QP]};
  }
  // k_i . k_j and q_i . k_j: accumulator register r = [i = 4 g + r][j = lo]
  f32x4 kk = {0.f, 0.f, 0.f, 0.f}, qk = kk;
#pragma unroll
  for (int dt = 0; dt < DT; ++dt) {
    const f32x4 ka = *reinterpret_cast<const f32x4*>(ks + lo * QP + dt * 16 + 4 * g);
    const f32x4 qa = *reinterpret_cast<const f32x4*>(qs + lo * QP + dt * 16 + 4 * g);
    kk = mfma_f32_k16(ka, ka, kk);
    qk = mfma_f32_k16(qa, ka, qk);
  }
  const int rep = a.H / G;
  float* Mw = M[wave];
  for (int hh = wave; hh < ((rep + 3) & ~3); hh += 4) {          // every wave makes the same number of turns
    const bool live = hh < rep;
    const int h = c * rep + (live ? hh : rep - 1);
    float* m = a.mats + (blk * a.H + h) * DELTA_MAT;
    // lane token lo: log decay, running sum over the tokens (all four groups of sixteen lanes alike), beta
    const long t = t0 + tb + min(lo, n - 1);
    float b = lo < n ? -expf(a.a_log[h]) * rec_softplus((float)((const T*)a.a_raw)[t * a.a_stride + h] + a.dt_bias[h]) : 0.f;
    const float beta = lo < n ? rec_sigmoid((float)((const T*)a.b_raw)[t * a.b_stride + h]) : 0.f;
#pragma unroll
    for (int o = 1; o < 16; o <<= 1) {
      const float up = __shfl(b, (lane & 48) | (lo >= o ? lo - o : lo), 64);
      if (lo >= o) b += up;
    }
    const float bn = __shfl(b, 15, 64);
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int i = 4 * g + r;
      const float bi = __shfl(b, i, 64), betai = __shfl(beta, i, 64);
      const float f = lo <= i ? expf(bi - b) : 0.f;
      Mw[i * 17 + lo] = lo < i ? betai * f * kk[r] : 0.f;
      if (live) m[256 + ((lo >> 2) * 16 + i) * 4 + (lo & 3)] = f * qk[r];
    }
    __syncthreads();
    // (I + M)^-1, one column per lane by forward substitution, times beta of the column
    float x[16];
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      float v = i == lo ? 1.f : 0.f;
#pragma unroll
      for (int j = 0; j < i; ++j) v -= Mw[i * 17 + j] * x[j];
      x[i] = v;
    }
    if (live && g == 0) {
#pragma unroll
      for (int i = 0; i < 16; ++i) m[((lo >> 2) * 16 + i) * 4 + (lo & 3)] = x[i] * beta;
      m[512 + lo] = expf(b);
      m[528 + lo] = expf(bn - b);
    }
    __syncthreads();
  }
}

// grid (H, sequences, groups of 64 columns): walks the blocks of its sequence, S of sixteen columns per wave in
// accumulators.  A block's operands (read by all four waves) sit in one of two LDS buffers while those of the next two
// blocks are on their way from memory; one barrier per block.  The column group is the slowest grid index, so that
// workgroups that read the same blocks tend to share an L2.
template <typename T, int DT>
__global__ __launch_bounds__(256) void delta_block_walk_kernel(const DeltaHeadArgs a) {
  constexpr int DP = DT * 16, NV = 48 * DP, BUF = NV + DELTA_MAT;
  constexpr int PF = (NV / 4 + 255) / 256;             // float4 of the vectors per thread and block
  extern __shared__ __align__(16) float lds[];
  const int srel = blockIdx.y, s = a.seq0 + srel, tid = threadIdx.x;
  const int lane = tid & 63, wave = tid >> 6, lo = lane & 15, g = lane >> 4;
  const int sl = a.seq_lens[s];
  if (sl <= 0) return;
  const int t0 = a.qsl[s], L = a.qsl[s + 1] - t0;
  if (L <= a.limit) return;
  const int h = blockIdx.x, D = a.D, Dv = a.Dv, H = a.H, G = a.G, c = h / (H / G);
  const int tile0 = blockIdx.z * 64 + wave * 16, col = tile0 + lo;
  const bool busy = tile0 < Dv, has_col = col < Dv;
  const bool vs4 = (D & 3) == 0;
  float* Scol = a.state + (((long)a.slot_table[s * a.st_stride] * H + h) * Dv + (has_col ? col : Dv - 1)) * (long)D;
  f32x4 S[DT];
  const bool carry = sl - L > 0;
#pragma unroll
  for (int dt = 0; dt < DT; ++dt) S[dt] = load4<float>(Scol + dt * 16 + 4 * g, carry ? D - dt * 16 - 4 * g : 0, vs4);
  const int nb = (L + 15) / 16;
  const long blk0 = (long)(t0 / 16) + srel;
  const T* vp = (const T*)a.qkv + (long)t0 * a.qkv_stride + (long)2 * G * D + (long)h * Dv + (has_col ? col : Dv - 1);

  const float* vec0 = a.vecs + (blk0 * G + c) * NV + tid * 4;
  const float* mat0 = a.mats + (blk0 * H + h) * DELTA_MAT + tid * 4;
  struct Fetched {
    f32x4 vec[PF], mat;
    T v[4];
  };
  auto fetch = [&](Fetched& f, int bi) {               // nothing here waits for the data
    const float* vp4 = vec0 + (long)bi * G * NV;
#pragma unroll
    for (int n = 0; n < PF; ++n)
      if ((n + 1) * 1024 <= NV || tid * 4 + n * 1024 < NV) f.vec[n] = *reinterpret_cast<const f32x4*>(vp4 + n * 1024);
    if (tid < DELTA_MAT / 4) f.mat = *reinterpret_cast<const f32x4*>(mat0 + (long)bi * H * DELTA_MAT);
#pragma unroll
    for (int r = 0; r < 4; ++r) f.v[r] = vp[(long)min(bi * 16 + 4 * g + r, L - 1) * a.qkv_stride];
  };
  f32x4 v;
  auto stage = [&](const Fetched& f, int bi) {         // block bi into its buffer, its values into v
    float* buf = lds + (bi & 1) * BUF;
#pragma unroll
    for (int n = 0; n < PF; ++n)
      if ((n + 1) * 1024 <= NV || tid * 4 + n * 1024 < NV) *reinterpret_cast<f32x4*>(buf + tid * 4 + n * 1024) = f.vec[n];
    if (tid < DELTA_MAT / 4) *reinterpret_cast<f32x4*>(buf + NV + tid * 4) = f.mat;
#pragma unroll
    for (int r = 0; r < 4; ++r) v[r] = bi * 16 + 4 * g + r < L ? (float)f.v[r] : 0.f;
  };
  auto run = [&](int bi) {
    const float* buf = lds + (bi & 1) * BUF;
    if (busy) {
      f32x4 ka = {0.f, 0.f, 0.f, 0.f}, kb = ka, qa = ka, qb = ka;
      // four accumulators in turn: a product never waits for the one right before it
#pragma unroll
      for (int dt = 0; dt < DT; dt += 2) {
        const f32x4 k0 = *reinterpret_cast<const f32x4*>(buf + (dt * 64 + lane) * 4);
        const f32x4 k1 = *reinterpret_cast<const f32x4*>(buf + (dt * 64 + 64 + lane) * 4);
        const f32x4 q0 = *reinterpret_cast<const f32x4*>(buf + 16 * DP + (dt * 64 + lane) * 4);
        const f32x4 q1 = *reinterpret_cast<const f32x4*>(buf + 16 * DP + (dt * 64 + 64 + lane) * 4);
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          ka = mfma_f32(k0[r], S[dt][r], ka);
          kb = mfma_f32(k1[r], S[dt + 1][r], kb);
          qa = mfma_f32(q0[r], S[dt][r], qa);
          qb = mfma_f32(q1[r], S[dt + 1][r], qb);
        }
      }
      const f32x4 tm = *reinterpret_cast<const f32x4*>(buf + NV + lane * 4);
      const f32x4 pm = *reinterpret_cast<const f32x4*>(buf + NV + 256 + lane * 4);
      const f32x4 eb = *reinterpret_cast<const f32x4*>(buf + NV + 512 + 4 * g);
      const f32x4 ek = *reinterpret_cast<const f32x4*>(buf + NV + 528 + 4 * g);
      const float en = buf[NV + 512 + 15];
      const f32x4 rhs = v - eb * (ka + kb);
      f32x4 u = {0.f, 0.f, 0.f, 0.f};
      u = mfma_f32_k16(tm, rhs, u);
      const f32x4 o = mfma_f32_k16(pm, u, eb * (qa + qb));
      u *= ek;
#pragma unroll
      for (int dt = 0; dt < DT; dt += 2) {
        const f32x4 kt0 = *reinterpret_cast<const f32x4*>(buf + 32 * DP + (dt * 64 + lane) * 4);
        const f32x4 kt1 = *reinterpret_cast<const f32x4*>(buf + 32 * DP + (dt * 64 + 64 + lane) * 4);
        S[dt] *= en;
        S[dt + 1] *= en;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          S[dt] = mfma_f32(kt0[r], u[r], S[dt]);
          S[dt + 1] = mfma_f32(kt1[r], u[r], S[dt + 1]);
        }
      }
      if (has_col) {
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int tt = bi * 16 + 4 * g + r;
          if (tt < L) a.o_raw[((long)(t0 + tt) * H + h) * Dv + col] = o[r];
        }
      }
    }
  };
  // two blocks ahead in registers, one ahead in LDS
  Fetched fa, fb;
  fetch(fa, 0);
  if (nb > 1) fetch(fb, 1);
  stage(fa, 0);
  __syncthreads();
  for (int bi = 0; bi < nb; bi += 2) {
    if (bi + 2 < nb) fetch(fa, bi + 2);
    run(bi);
    if (bi + 1 < nb) stage(fb, bi + 1);
    __syncthreads();
    if (bi + 1 < nb) {
      if (bi + 3 < nb) fetch(fb, bi + 3);
      run(bi + 1);
      if (bi + 2 < nb) stage(fa, bi + 2);
      __syncthreads();
    }
  }
  if (has_col) {
#pragma unroll
    for (int dt = 0; dt < DT; ++dt) store4(Scol + dt * 16 + 4 * g, S[dt], D - dt * 16 - 4 * g, vs4);
  }
}

static int delta_dt(int D) { return D <= 32 ? 2 : D <= 64 ? 4 : D <= 128 ? 8 : 16; }

// floats of scratch the chunked form needs for T tokens of S sequences
VDA_EXPORT long vda_delta_head_scratch(int T, int S, int H, int G, int D) {
  const long blocks = (long)T / 16 + S + 1;
  return blocks * ((long)G * 3 * 16 * delta_dt(D) * 16 + (long)H * DELTA_MAT);
}

VDA_EXPORT int vda_gated_delta_rule_head(void* out, long o_stride, float* o_raw, float* scratch, const void* qkv,
                                         long qkv_stride, const void* a_raw, long a_stride, const void* b_raw,
                                         long b_stride, const void* gate, long g_stride, const float* a_log,
                                         const float* dt_bias, const float* norm_w, float* state, const int* qsl,
                                         const int* seq_lens, const int* slot_table, long st_stride, int T, int S,
                                         int seq0, int H, int G, int D, int Dv, int max_q, float eps, int dtype,
                                         hipStream_t st) {
  if (S <= 0 || T <= 0) return 0;
  if (H <= 0 || G <= 0 || H % G || D < 1 || D > 1024 || Dv < 1 || seq0 < 0 || seq0 > S) return -1;
  const bool chunked = D <= 256 && max_q > 16 && scratch && o_raw && seq0 < S;
  DeltaHeadArgs a;
  a.qkv = qkv; a.qkv_stride = qkv_stride; a.a_raw = a_raw; a.b_raw = b_raw; a.gate = gate; a.a_stride = a_stride;
  a.b_stride = b_stride; a.g_stride = g_stride; a.a_log = a_log; a.dt_bias = dt_bias; a.norm_w = norm_w; a.eps = eps;
  a.state = state; a.out = out; a.o_stride = o_stride; a.o_raw = o_raw; a.qsl = qsl; a.seq_lens = seq_lens;
  a.slot_table = slot_table; a.st_stride = st_stride; a.H = H; a.G = G; a.D = D; a.Dv = Dv; a.seq0 = seq0;
  a.limit = chunked ? 16 : 0x7fffffff;
  const int DT = delta_dt(D);
  const long blocks = (long)T / 16 + (S - seq0) + 1;
  a.vecs = scratch;
  a.mats = scratch ? scratch + blocks * G * 48 * (DT * 16) : nullptr;
  int NR = 1;
  while (16 * NR < D) NR *= 2;
  int tile = max_q < 16 ? max_q : 16;
  auto step_lds = [&](int tl) { return ((size_t)tl * 2 * 16 * NR + (size_t)2 * tl * Dv + 4 * tl) * 4; };
  while (tile > 1 && step_lds(tile) > 48 * 1024) tile >>= 1;
  if (step_lds(tile) > 60 * 1024) return -2;
  const size_t slds = step_lds(tile);
#define STEP(TT, NN) hipLaunchKernelGGL((delta_step_kernel<TT, NN>), dim3(H, S), dim3(256), slds, st, a, tile)
#define STEPS(TT)                                                                                                      \
  switch (NR) {                                                                                                        \
    case 1: STEP(TT, 1); break;                                                                                        \
    case 2: STEP(TT, 2); break;                                                                                        \
    case 4: STEP(TT, 4); break;                                                                                        \
    case 8: STEP(TT, 8); break;                                                                                        \
    case 16: STEP(TT, 16); break;                                                                                      \
    case 32: STEP(TT, 32); break;                                                                                      \
    default: STEP(TT, 64); break;                                                                                      \
  }
  if (dtype == VDA_BF16) { STEPS(bf16_t) }
  else if (dtype == VDA_F16) { STEPS(f16_t) }
  else if (dtype == VDA_F32) { STEPS(float) }
  else return -3;
#undef STEPS
#undef STEP
  VDA_CHECK_LAUNCH();
  if (!chunked) return 0;
  const dim3 gp((max_q + 15) / 16, S - seq0, G), gw(H, S - seq0, (Dv + 63) / 64);
  const size_t wlds = (size_t)2 * (48 * DT * 16 + DELTA_MAT) * 4;
#define CK(TT, DD)                                                                                                     \
  do {                                                                                                                 \
    if (wlds > 48 * 1024) {                                                                                            \
      hipError_t e_ = hipFuncSetAttribute((const void*)delta_block_walk_kernel<TT, DD>,                                \
                                          hipFuncAttributeMaxDynamicSharedMemorySize, (int)wlds);                      \
      if (e_ != hipSuccess) return (int)e_;                                                                            \
    }                                                                                                                  \
    hipLaunchKernelGGL((delta_block_prepare_kernel<TT, DD>), gp, dim3(256), 0, st, a);                                 \
    hipLaunchKernelGGL((delta_block_walk_kernel<TT, DD>), gw, dim3(256), wlds, st, a);                                 \
  } while (0)
#define CA(TT) do { if (DT == 2) CK(TT, 2); else if (DT == 4) CK(TT, 4); else if (DT == 8) CK(TT, 8); else CK(TT, 16); } while (0)
  if (dtype == VDA_BF16) CA(bf16_t);
  else if (dtype == VDA_F16) CA(f16_t);
  else CA(float);
#undef CA
#undef CK
  VDA_CHECK_LAUNCH();
  const dim3 ge((unsigned)(((long)max_q * H + 3) / 4), S - seq0);
#define EP(TT) hipLaunchKernelGGL((head_norm_silu_kernel<TT>), ge, dim3(256), 0, st, (TT*)out, o_stride, o_raw,        \
                                  (const TT*)gate, g_stride, norm_w, 0, qsl, seq_lens, seq0, a.limit, H, Dv, eps)
  if (dtype == VDA_BF16) EP(bf16_t);
  else if (dtype == VDA_F16) EP(f16_t);
  else EP(float);
#undef EP
  VDA_CHECK_LAUNCH();
  return 0;
}
