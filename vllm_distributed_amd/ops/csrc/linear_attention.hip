// Linear attention with decay over a ragged batch with per-request fp32 state.  Per token and head
//     S <- diag(decay) S + k v^T,   o = S^T q                       (S: [D, Dv], stored transposed, [Dv, D])
//     out = o / rms(o) * norm_w * silu(gate)                        (norm_w optional)
// or, with a bonus u per head and key channel (the RWKV form: the own token enters the read-out through the bonus, not the
// memory),   o = (S + diag(u) k v^T)^T q,   S <- diag(decay) S + k v^T,
// with q and k scaled and, on the first `rot` values of a head, rotated (value i paired with i + rot / 2, fp32 angles from
// a table) before they enter, and a decay that is either
//     one number per head (retention):              decay[h], given as its logarithm, or
//     one number per token, head and key channel:   sigmoid(z + bias)^(1 / tau) (gated linear attention), or
//                                                   exp(-exp(z + bias)) (`decay_exp`).
// The batch description is the one of the other recurrent kernels (qsl, seq_lens, slot in column 0 of the table; a
// sequence carries state in when seq_len - new_tokens > 0).
//
// Sequences with few new tokens (decoding, short portions):
//   step   one workgroup per (sequence, head), token by token, everything in one launch: the state is read and written
//          once, norm and gate included.
// Longer ones (when the rows allow 4-value accesses; otherwise `step` walks them too), chunk-parallel on the fp32 matrix
// instruction (recurrent.h), a sequence cut into chunks of C tokens:
//   chunk<OUT = false>   per (chunk, head): the state the chunk alone would build, and its total decay
//   carry                per (sequence, head): the state at every chunk's start, one after the other (elementwise)
//   chunk<OUT = true>    per (chunk, head): from that state, sixteen tokens at a time:
//                            o_i = (q_i e^b_i)^T S + sum over j <= i of (sum_d q_id k_jd e^(b_id - b_jd)) v_j
//                            with a bonus: b_(i-1) in the place of b_i, j < i, and (sum_d q_id u_d k_id) v_i on top
//                            S  <- diag(e^b_n) S + sum_j (k_j e^(b_n - b_j)) v_j^T        b: running sum of log decays
//                        norm and gate in the same launch when one workgroup holds all of a head's columns.
// Every exponent that is formed is <= 0 but one: e^-b_j, used only while the sixteen tokens' b stays above -40; stronger
// decays take the product element by element.
#include "recurrent.h"

struct LinArgs {
  const void *q, *k, *v, *z, *gate;
  long q_stride, k_stride, v_stride, z_stride, g_stride;
  const float* z_bias;          // [H * D] or null
  float inv_tau;
  int decay_exp;                // decay exp(-exp(z + bias)) instead of sigmoid(z + bias)^inv_tau
  const float* bonus;           // [H * D] or null (with z only)
  const float* log_decay;       // [H] (no z)
  const float* cos_sin;         // [positions, rot]
  const long* positions;
  int rot;
  float q_scale, k_scale;
  const float* norm_w;          // [Dv], [H * Dv] (norm_head = Dv) or null
  int norm_head;                // values between two heads' norm weights
  float eps;
  float* state;                 // [slots, H, Dv, D]
  void* out;
  long o_stride;
  float* o_raw;                 // [T, H * Dv] fp32 when norm and gate run in a launch of their own, else null
  const int *qsl, *seq_lens, *slot_table;
  long st_stride;
  int H, D, Dv;
  int seq0;                     // first sequence of the chunk kernels
  int C;                        // tokens per chunk (multiple of 16)
  float* chunk_state;           // [chunks, H, column tiles, DT, 64 lanes, 4]
  float* chunk_decay;           // [chunks, H, DP] (channel decays)
  int limit;                    // sequences with at most this many new tokens belong to `step`, others to `chunk`
  int col_groups;
  int vec;                      // D % 4 == 0 and all q / k / z rows aligned for 4-value loads
};

// values d .. d + 3 of a q or k row of head h at token t: rotated, unscaled, zeros from D on
template <typename T>
__device__ __forceinline__ f32x4 lin_row4(const LinArgs& a, const T* row, int d, long t) {
  f32x4 x = load4<T>(row + d, a.D - d, a.vec);
  if (a.rot > 0 && d < a.rot) {
    const int half = a.rot >> 1;
    const float* cs = a.cos_sin + a.positions[t] * (long)a.rot;
    if (a.vec && (half & 3) == 0) {
      const bool low = d < half;
      const f32x4 o = load4<T>(row + (low ? d + half : d - half), 4, true);
      const float* cp = cs + (low ? d : d - half);
      const f32x4 c = {cp[0], cp[1], cp[2], cp[3]}, s = {cp[half], cp[half + 1], cp[half + 2], cp[half + 3]};
#pragma unroll
      for (int i = 0; i < 4; ++i) x[i] = low ? x[i] * c[i] - o[i] * s[i] : x[i] * c[i] + o[i] * s[i];
    } else {
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int dd = d + i;
        if (dd < a.rot) {
          const bool low = dd < half;
          const float o = (float)row[low ? dd + half : dd - half];
          const int ci = low ? dd : dd - half;
          x[i] = low ? x[i] * cs[ci] - o * cs[half + ci] : x[i] * cs[ci] + o * cs[half + ci];
        }
      }
    }
  }
  return x;
}

// log decay of a channel whose pre-activation is z.  exp(-exp(z)) is zero in fp32 long before the bound, which keeps
// differences of running sums finite and exact.
__device__ __forceinline__ float lin_log_decay(const LinArgs& a, float z) {
  return a.decay_exp ? fmaxf(-expf(z), -200.f) : rec_logsigmoid(z) * a.inv_tau;
}

// log decays of channels d .. d + 3 at token t (0 beyond D)
template <typename T>
__device__ __forceinline__ f32x4 lin_log_decay4(const LinArgs& a, long t, int h, int d) {
  f32x4 o = {0.f, 0.f, 0.f, 0.f};
  const int n = a.D - d;
  if (n <= 0) return o;
  const f32x4 z = load4<T>((const T*)a.z + t * a.z_stride + (long)h * a.D + d, n, a.vec);
#pragma unroll
  for (int i = 0; i < 4; ++i)
    if (i < n) o[i] = lin_log_decay(a, z[i] + (a.z_bias ? a.z_bias[(long)h * a.D + d + i] : 0.f));
  return o;
}

// ---- few new tokens ------------------------------------------------------------------------------------------------
// grid (H, S); 16 columns x 16 lanes at a time, NCG such column groups in registers together
template <typename T, int NR, bool CHAN, bool BONUS>
__global__ __launch_bounds__(256) void lin_step_kernel(const LinArgs a, const int tile) {
  constexpr int NCG = NR <= 8 ? 4 : NR <= 16 ? 2 : 1;
  constexpr int DP = 16 * NR;
  extern __shared__ __align__(16) float lds[];
  const int h = blockIdx.x, s = blockIdx.y, tid = threadIdx.x;
  const int sl = a.seq_lens[s];
  if (sl <= 0) return;
  const int t0 = a.qsl[s], L = a.qsl[s + 1] - t0;
  if (L <= 0 || L > a.limit) return;
  const int D = a.D, Dv = a.Dv;
  float* qs = lds;                                     // [tile][DP]
  float* ks = qs + tile * DP;
  float* gs = ks + tile * DP;                          // CHAN only
  float* vs = gs + (CHAN ? tile * DP : 0);             // [tile][Dv]
  float* os = vs + tile * Dv;                          // [tile][Dv]
  const int part = tid & 15, sub = tid >> 4, lane = tid & 63, wave = tid >> 6;
  const bool carry = sl - L > 0;
  const bool vs4 = (D & 3) == 0;
  float* Sb = a.state + ((long)a.slot_table[s * a.st_stride] * a.H + h) * (long)Dv * D;
  const float gh = CHAN ? 0.f : expf(a.log_decay[h]);
  float S[NCG][NR], ur[NR];
  if (BONUS) {
#pragma unroll
    for (int i = 0; i < NR; ++i) {
      const int d = rec_lane_value<NR>(part, i);
      ur[i] = d < D ? a.bonus[(long)h * D + d] : 0.f;
    }
  }
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
    for (int e = tid; e < nt * (DP / 4); e += 256) {
      const int tt = e / (DP / 4), d = (e - tt * (DP / 4)) * 4;
      const long t = t0 + b + tt;
      const f32x4 q = lin_row4<T>(a, (const T*)a.q + t * a.q_stride + (long)h * D, d, t);
      const f32x4 k = lin_row4<T>(a, (const T*)a.k + t * a.k_stride + (long)h * D, d, t);
      f32x4 g = {0.f, 0.f, 0.f, 0.f};
      if (CHAN) {
        g = lin_log_decay4<T>(a, t, h, d);
#pragma unroll
        for (int i = 0; i < 4; ++i) g[i] = expf(g[i]);
        *reinterpret_cast<f32x4*>(gs + tt * DP + d) = g;
      }
      *reinterpret_cast<f32x4*>(qs + tt * DP + d) = q * a.q_scale;
      *reinterpret_cast<f32x4*>(ks + tt * DP + d) = k * a.k_scale;
    }
    for (int e = tid; e < nt * Dv; e += 256) {
      const int tt = e / Dv, c = e - tt * Dv;
      vs[e] = (float)((const T*)a.v)[(long)(t0 + b + tt) * a.v_stride + (long)h * Dv + c];
    }
    __syncthreads();
    for (int c0 = 0; c0 < Dv; c0 += 16 * NCG) {
      for (int tt = 0; tt < nt; ++tt) {
        float kr[NR], qr[NR], gr[NR];
        rec_lane_row<NR>(kr, ks + tt * DP, part);
        rec_lane_row<NR>(qr, qs + tt * DP, part);
        if (CHAN) rec_lane_row<NR>(gr, gs + tt * DP, part);
#pragma unroll
        for (int n = 0; n < NCG; ++n) {
          const int col = c0 + n * 16 + sub;
          const float v = vs[tt * Dv + (col < Dv ? col : Dv - 1)];
          float p = 0.f;
#pragma unroll
          for (int i = 0; i < NR; ++i) {
            const float kv = kr[i] * v;
            if (BONUS) p += (S[n][i] + ur[i] * kv) * qr[i];
            S[n][i] = S[n][i] * (CHAN ? gr[i] : gh) + kv;
            if (!BONUS) p += S[n][i] * qr[i];
          }
          p = row16_sum(p);
          if (part == 0 && col < Dv) os[tt * Dv + col] = p;
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
      for (int c = lane; c < Dv; c += 64) ss += o[c] * o[c];
      ss = wave_sum(ss);
      const float rs = 1.f / sqrtf(ss / (float)Dv + a.eps);
      for (int c = lane; c < Dv; c += 64) {
        const float zg = (float)((const T*)a.gate)[t * a.g_stride + (long)h * Dv + c];
        ((T*)a.out)[t * a.o_stride + (long)h * Dv + c] =
            (T)(o[c] * rs * (a.norm_w ? a.norm_w[(long)h * a.norm_head + c] : 1.f) * zg * rec_sigmoid(zg));
      }
    }
  }
}

// ---- chunk-parallel form -------------------------------------------------------------------------------------------
// grid (chunks of the longest sequence, sequences, heads x column groups); wave w holds columns
// (w * ET .. w * ET + ET - 1) * 16 of the group, all D rows of them in accumulators.  Rows are aligned for 4-value
// accesses and D, Dv and rot / 2 are multiples of 4.
// Staging layout: thread -> token tid / 16, values d0 + 64 m with d0 = 4 * (tid % 16).  The next sixteen tokens' rows are
// on their way from memory, unconverted, while these are computed; a block's output leaves LDS in the staging phase of
// the next one, so two barriers (four with channel decays) separate everything.
template <typename T, int DT, int ET, bool CHAN, bool OUT, bool BONUS>
__global__ __launch_bounds__(256, DT <= 4 ? 3 : DT == 8 ? 2 : 1) void lin_chunk_kernel(const LinArgs a) {
  constexpr int DP = DT * 16, QP = DP + 4, TP = 20, CW = 64 * ET, OP = CW + 4;
  constexpr int NI = (DP + 63) / 64, NVI = ET;
  using V4 = typename Vec<T>::v4;
  extern __shared__ __align__(16) float lds[];
  float* ks = lds;                                     // [16][QP]
  float* kT = ks + 16 * QP;                            // [DP][TP]   k_j e^(b_n - b_j), transposed
  float* vT = kT + DP * TP;                            // [CW][TP]
  float* qs = vT + CW * TP;                            // [16][QP]   (OUT)
  float* os = qs + (OUT ? 16 * QP : 0);                // [16][OP]   (OUT)
  float* bc = os + (OUT ? 16 * OP : 0);                // [16][QP]   (CHAN) running sums of log decays
  float* dec = bc + (CHAN ? 16 * QP : 0);              // [DP]       (CHAN) e^b_n
  float* bon = dec + (CHAN ? DP : 0);                  // [16]       (BONUS) sum_d q u k of each token
  const int srel = blockIdx.y, s = a.seq0 + srel, tid = threadIdx.x;
  const int sl = a.seq_lens[s];
  if (sl <= 0) return;
  const int t0 = a.qsl[s], L = a.qsl[s + 1] - t0;
  if (L <= a.limit) return;
  const int C = a.C, nch = (L + C - 1) / C, c = blockIdx.x;
  if (c >= nch || (!OUT && c == nch - 1)) return;
  const int D = a.D, Dv = a.Dv, H = a.H;
  const int h = blockIdx.z / a.col_groups, cg = blockIdx.z - h * a.col_groups;
  const int lane = tid & 63, wave = tid >> 6, lo = lane & 15, g = lane >> 4;
  const int coltiles = (Dv + 15) / 16;
  const int tile0 = cg * 4 * ET + wave * ET;           // this wave's first column tile
  const int col0 = cg * CW;                            // the workgroup's first column
  const bool busy = tile0 < coltiles;
  const long cidx = ((long)(t0 / C) + srel + c) * H + h;
  float* cst = a.chunk_state + cidx * coltiles * (DT * 256);
  float* Sb = a.state + ((long)a.slot_table[s * a.st_stride] * H + h) * (long)Dv * D;
  f32x4 S[ET][DT];
  const bool from_chunk = OUT && nch > 1, from_slot = OUT && nch == 1 && sl - L > 0;
#pragma unroll
  for (int e = 0; e < ET; ++e) {
    const int ct = tile0 + e, col = ct * 16 + lo;
#pragma unroll
    for (int dt = 0; dt < DT; ++dt) {
      const int d = dt * 16 + 4 * g;
      S[e][dt] = f32x4{0.f, 0.f, 0.f, 0.f};
      if (from_chunk && ct < coltiles) S[e][dt] = *reinterpret_cast<const f32x4*>(cst + ((ct * DT + dt) * 64 + lane) * 4);
      if (from_slot && col < Dv && d < D) S[e][dt] = *reinterpret_cast<const f32x4*>(Sb + (long)col * D + d);
    }
  }
  const float ld = CHAN ? 0.f : a.log_decay[h];
  float tot = 0.f;                                     // CHAN, thread d: sum of channel d's log decays over the chunk
  float pf[4], of[4];                                  // e^(b_i - b_j) of this lane's pairs, e^b_i of its rows
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    pf[r] = 4 * g + r <= lo ? expf(ld * (float)(lo - 4 * g - r)) : 0.f;
    of[r] = expf(ld * (float)(4 * g + r + 1));
  }
  const int tt = tid >> 4, d0 = (tid & 15) * 4, half = a.rot >> 1;
  const T* kp = (const T*)a.k + (long)h * D + t0 * a.k_stride;
  const T* qp = (const T*)a.q + (long)h * D + t0 * a.q_stride;
  const T* vp = (const T*)a.v + (long)h * Dv + t0 * a.v_stride + col0;
  const T* zp = CHAN ? (const T*)a.z + (long)h * D + t0 * a.z_stride : nullptr;
  const T* gp = (const T*)a.gate + (long)h * Dv + t0 * a.g_stride;
  V4 rk[NI], rk2[NI], rq[NI], rq2[NI], rz[NI], rv[NVI], rg[NVI];
  f32x4 ru[NI];
  if (BONUS && OUT) {
#pragma unroll
    for (int m = 0; m < NI; ++m)
      ru[m] = *reinterpret_cast<const f32x4*>(a.bonus + (long)h * D + (d0 + 64 * m < D ? d0 + 64 * m : 0));
  }
  int pos = 0;
  auto fetch = [&](int tb) {
    const long t = min(tb + tt, L - 1);
    if (!CHAN && a.rot > 0) pos = (int)a.positions[t0 + t];
#pragma unroll
    for (int m = 0; m < NI; ++m) {
      const int d = d0 + 64 * m, dc = d < D ? d : 0;
      rk[m] = *reinterpret_cast<const V4*>(kp + t * a.k_stride + dc);
      if (OUT) rq[m] = *reinterpret_cast<const V4*>(qp + t * a.q_stride + dc);
      if (CHAN) rz[m] = *reinterpret_cast<const V4*>(zp + t * a.z_stride + dc);
      if (!CHAN && a.rot > 0) {
        const int dp = d < a.rot ? (d < half ? d + half : d - half) : dc;
        rk2[m] = *reinterpret_cast<const V4*>(kp + t * a.k_stride + dp);
        if (OUT) rq2[m] = *reinterpret_cast<const V4*>(qp + t * a.q_stride + dp);
      }
    }
#pragma unroll
    for (int m = 0; m < NVI; ++m) {
      const int cc = d0 + 64 * m;
      rv[m] = *reinterpret_cast<const V4*>(vp + t * a.v_stride + (col0 + cc < Dv ? cc : 0));
    }
  };
  // rows tb .. tb + 15 of the output: norm over the head's columns, weight, gate (or the plain sums)
  auto emit = [&](int tb) {
    if (tb + tt >= min(L, c * C + C)) return;
    const long t = tb + tt;
    f32x4 o[NVI];
    float ss = 0.f;
#pragma unroll
    for (int m = 0; m < NVI; ++m) {
      o[m] = f32x4{0.f, 0.f, 0.f, 0.f};
      if (col0 + d0 + 64 * m < Dv) o[m] = *reinterpret_cast<const f32x4*>(os + tt * OP + d0 + 64 * m);
      ss += o[m][0] * o[m][0] + o[m][1] * o[m][1] + o[m][2] * o[m][2] + o[m][3] * o[m][3];
    }
    if (a.o_raw) {
#pragma unroll
      for (int m = 0; m < NVI; ++m)
        if (col0 + d0 + 64 * m < Dv)
          *reinterpret_cast<f32x4*>(a.o_raw + ((t0 + t) * H + h) * Dv + col0 + d0 + 64 * m) = o[m];
      return;
    }
    ss = row16_sum(ss);                                // a token's columns sit in sixteen neighbouring lanes
    const float rs = 1.f / sqrtf(ss / (float)Dv + a.eps);
#pragma unroll
    for (int m = 0; m < NVI; ++m) {
      const int cc = d0 + 64 * m;
      if (cc >= Dv) continue;
      f32x4 w = {1.f, 1.f, 1.f, 1.f};
      if (a.norm_w) w = *reinterpret_cast<const f32x4*>(a.norm_w + (long)h * a.norm_head + cc);
      V4 y;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const float zg = (float)rg[m][i];
        y[i] = (T)(o[m][i] * rs * w[i] * zg * rec_sigmoid(zg));
      }
      *reinterpret_cast<V4*>((T*)a.out + (t0 + t) * a.o_stride + (long)h * Dv + cc) = y;
    }
  };
  const int first = c * C, end = min(L, first + C);
  fetch(first);
  for (int tb = first; tb < end; tb += 16) {
    const int n = min(16, end - tb);
    const bool on = tt < n;
    f32x4 rc[NI], rs[NI];
    if (!CHAN && a.rot > 0) {
      const float* cs = a.cos_sin + pos * (long)a.rot;
#pragma unroll
      for (int m = 0; m < NI; ++m) {
        const int d = d0 + 64 * m, ci = d < a.rot ? (d < half ? d : d - half) : 0;
        rc[m] = *reinterpret_cast<const f32x4*>(cs + ci);
        rs[m] = *reinterpret_cast<const f32x4*>(cs + half + ci);
      }
    }
    __syncthreads();
    if (OUT && tb > first) emit(tb - 16);
    const float f = CHAN ? 0.f : expf(ld * (float)max(n - 1 - tt, 0));
    float quk = 0.f;
#pragma unroll
    for (int m = 0; m < NI; ++m) {
      const int d = d0 + 64 * m;
      if (DP < 64 && d >= DP) continue;
      f32x4 k, q = {0.f, 0.f, 0.f, 0.f}, b = q;
      const bool live = on && d < D, turn = !CHAN && d < a.rot;
      const float sg = d < half ? -1.f : 1.f;
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        float y = (float)rk[m][i];
        if (turn) y = y * rc[m][i] + sg * (float)rk2[m][i] * rs[m][i];
        k[i] = live ? y * a.k_scale : 0.f;
        if (OUT) {
          float x = (float)rq[m][i];
          if (turn) x = x * rc[m][i] + sg * (float)rq2[m][i] * rs[m][i];
          q[i] = live ? x * a.q_scale : 0.f;
        }
      }
      *reinterpret_cast<f32x4*>(ks + tt * QP + d) = k;
      if (OUT) *reinterpret_cast<f32x4*>(qs + tt * QP + d) = q;
      if (BONUS && OUT) quk += q[0] * k[0] * ru[m][0] + q[1] * k[1] * ru[m][1] + q[2] * k[2] * ru[m][2] + q[3] * k[3] * ru[m][3];
      if (CHAN) {
        if (live) {
          f32x4 zb = {0.f, 0.f, 0.f, 0.f};
          if (a.z_bias) zb = *reinterpret_cast<const f32x4*>(a.z_bias + (long)h * D + d);
#pragma unroll
          for (int i = 0; i < 4; ++i) b[i] = lin_log_decay(a, (float)rz[m][i] + zb[i]);
        }
        *reinterpret_cast<f32x4*>(bc + tt * QP + d) = b;
      } else {
#pragma unroll
        for (int i = 0; i < 4; ++i) kT[(d + i) * TP + tt] = k[i] * f;
      }
    }
    if (BONUS && OUT) {                                // a token's values sit in sixteen neighbouring lanes
      quk = row16_sum(quk);
      if ((tid & 15) == 0) bon[tt] = quk;
    }
#pragma unroll
    for (int m = 0; m < NVI; ++m) {
      const int cc = d0 + 64 * m;
      const bool live = on && col0 + cc < Dv;
#pragma unroll
      for (int i = 0; i < 4; ++i) vT[(cc + i) * TP + tt] = live ? (float)rv[m][i] : 0.f;
    }
    if (OUT && !a.o_raw) {                             // this block's gates; used when its output leaves
      const long t = min(tb + tt, L - 1);
#pragma unroll
      for (int m = 0; m < NVI; ++m) {
        const int cc = d0 + 64 * m;
        rg[m] = *reinterpret_cast<const V4*>(gp + t * a.g_stride + (cc < Dv ? cc : 0));
      }
    }
    if (tb + 16 < end) fetch(tb + 16);
    __syncthreads();
    f32x4 pt = {0.f, 0.f, 0.f, 0.f}, pt2 = pt;         // P^T: [j = 4 g + r][i = lo]
    int strong = 0;
    if (CHAN) {
      if (tid < DP) {
        float run[16];
#pragma unroll
        for (int j = 0; j < 16; ++j) run[j] = bc[j * QP + tid];
#pragma unroll
        for (int j = 1; j < 16; ++j) run[j] += run[j - 1];
#pragma unroll
        for (int j = 0; j < 16; ++j) bc[j * QP + tid] = run[j];
        dec[tid] = expf(run[15]);
        tot += run[15];
        strong = run[15] < -40.f;
      }
      strong = __syncthreads_or(strong);
      if (OUT && strong) {
        // element by element, all exponents <= 0
        if (busy) {
          for (int d = 0; d < D; ++d) {
            const float qi = qs[lo * QP + d], bi = BONUS ? (lo ? bc[(lo - 1) * QP + d] : 0.f) : bc[lo * QP + d];
#pragma unroll
            for (int r = 0; r < 4; ++r) {
              const int j = 4 * g + r;
              pt[r] += j <= lo - (BONUS ? 1 : 0) ? qi * ks[j * QP + d] * expf(bi - bc[j * QP + d]) : 0.f;
            }
          }
        }
        __syncthreads();
      }
#pragma unroll
      for (int m = 0; m < NI; ++m) {
        const int d = d0 + 64 * m;
        if (DP < 64 && d >= DP) continue;
        const f32x4 b = *reinterpret_cast<const f32x4*>(bc + tt * QP + d);
        const f32x4 bn = *reinterpret_cast<const f32x4*>(bc + 15 * QP + d);
        f32x4 k = *reinterpret_cast<const f32x4*>(ks + tt * QP + d);
#pragma unroll
        for (int i = 0; i < 4; ++i) kT[(d + i) * TP + tt] = k[i] * expf(bn[i] - b[i]);
        if (OUT) {
          f32x4 q = *reinterpret_cast<const f32x4*>(qs + tt * QP + d);
          f32x4 bq = b;                                // the decays between the state's time and the read-out
          if (BONUS) bq = tt ? *reinterpret_cast<const f32x4*>(bc + (tt - 1) * QP + d) : f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            q[i] *= expf(bq[i]);
            if (!strong) k[i] *= expf(-b[i]);
          }
          *reinterpret_cast<f32x4*>(qs + tt * QP + d) = q;
          if (!strong) *reinterpret_cast<f32x4*>(ks + tt * QP + d) = k;
        }
      }
      __syncthreads();
    }
    if (!busy) continue;
    f32x4 v4[ET];
#pragma unroll
    for (int e = 0; e < ET; ++e) v4[e] = *reinterpret_cast<const f32x4*>(vT + ((wave * ET + e) * 16 + lo) * TP + 4 * g);
    if (OUT) {
      if (!CHAN || !strong) {
#pragma unroll
        for (int dt = 0; dt < DT; dt += 2) {
          const float* kr = ks + lo * QP + dt * 16 + 4 * g;
          const float* qr = qs + lo * QP + dt * 16 + 4 * g;
          mfma_f32_k16_two(*(const f32x4*)kr, *(const f32x4*)qr, pt, *(const f32x4*)(kr + 16), *(const f32x4*)(qr + 16), pt2);
        }
        pt += pt2;
#pragma unroll
        for (int r = 0; r < 4; ++r) pt[r] = CHAN ? (4 * g + r <= lo ? pt[r] : 0.f) : pt[r] * pf[r];
      }
      if (BONUS) {
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (4 * g + r == lo) pt[r] = bon[lo];
      }
      f32x4 O[ET], o2[ET];
#pragma unroll
      for (int e = 0; e < ET; ++e) O[e] = o2[e] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int dt = 0; dt < DT; dt += 2) {
        const f32x4 q0 = *reinterpret_cast<const f32x4*>(qs + lo * QP + dt * 16 + 4 * g);
        const f32x4 q1 = *reinterpret_cast<const f32x4*>(qs + lo * QP + dt * 16 + 16 + 4 * g);
#pragma unroll
        for (int r = 0; r < 4; ++r)
#pragma unroll
          for (int e = 0; e < ET; ++e) {
            O[e] = mfma_f32(q0[r], S[e][dt][r], O[e]);
            o2[e] = mfma_f32(q1[r], S[e][dt + 1][r], o2[e]);
          }
      }
#pragma unroll
      for (int e = 0; e < ET; ++e) {
        O[e] += o2[e];
        if (!CHAN) {
#pragma unroll
          for (int r = 0; r < 4; ++r) O[e][r] *= of[r];
        }
        O[e] = mfma_f32_k16(pt, v4[e], O[e]);
#pragma unroll
        for (int r = 0; r < 4; ++r) os[(4 * g + r) * OP + (wave * ET + e) * 16 + lo] = O[e][r];
      }
    }
    const float dn = CHAN ? 0.f : expf(ld * (float)n);
#pragma unroll
    for (int dt = 0; dt < DT; dt += 2) {
      const f32x4 k0 = *reinterpret_cast<const f32x4*>(kT + (dt * 16 + lo) * TP + 4 * g);
      const f32x4 k1 = *reinterpret_cast<const f32x4*>(kT + (dt * 16 + 16 + lo) * TP + 4 * g);
      f32x4 g0 = {dn, dn, dn, dn}, g1 = g0;
      if (CHAN) {
        g0 = *reinterpret_cast<const f32x4*>(dec + dt * 16 + 4 * g);
        g1 = *reinterpret_cast<const f32x4*>(dec + dt * 16 + 16 + 4 * g);
      }
#pragma unroll
      for (int e = 0; e < ET; ++e) {
        S[e][dt] *= g0;
        S[e][dt + 1] *= g1;
      }
#pragma unroll
      for (int r = 0; r < 4; ++r)
#pragma unroll
        for (int e = 0; e < ET; ++e) {
          S[e][dt] = mfma_f32(k0[r], v4[e][r], S[e][dt]);
          S[e][dt + 1] = mfma_f32(k1[r], v4[e][r], S[e][dt + 1]);
        }
    }
  }
  if (OUT) {
    __syncthreads();
    emit((end - 1 - first) / 16 * 16 + first);
    if (c != nch - 1) return;
  } else if (CHAN && cg == 0 && tid < DP) {
    a.chunk_decay[cidx * DP + tid] = expf(tot);
  }
#pragma unroll
  for (int e = 0; e < ET; ++e) {
    const int ct = tile0 + e, col = ct * 16 + lo;
#pragma unroll
    for (int dt = 0; dt < DT; ++dt) {
      const int d = dt * 16 + 4 * g;
      if (!OUT && ct < coltiles) *reinterpret_cast<f32x4*>(cst + ((ct * DT + dt) * 64 + lane) * 4) = S[e][dt];
      if (OUT && col < Dv && d < D) *reinterpret_cast<f32x4*>(Sb + (long)col * D + d) = S[e][dt];
    }
  }
}

// what a chunk alone built -> the state at its start, chunk after chunk; four values per thread
template <bool CHAN>
__global__ __launch_bounds__(256) void lin_carry_kernel(const LinArgs a, const int DT) {
  const int srel = blockIdx.y, s = a.seq0 + srel;
  const int sl = a.seq_lens[s];
  if (sl <= 0) return;
  const int t0 = a.qsl[s], L = a.qsl[s + 1] - t0;
  if (L <= a.limit) return;
  const int C = a.C, nch = (L + C - 1) / C;
  if (nch <= 1) return;
  const int D = a.D, Dv = a.Dv, H = a.H, DP = DT * 16, coltiles = (Dv + 15) / 16;
  const int per = coltiles * DT * 64;                  // float4 per (chunk, head)
  const int i = blockIdx.x * 256 + threadIdx.x, h = blockIdx.z;
  if (i >= per) return;
  const int lane = i & 63, dt = (i >> 6) % DT, ct = (i >> 6) / DT;
  const int d = dt * 16 + 4 * (lane >> 4), col = ct * 16 + (lane & 15);
  f32x4 S = {0.f, 0.f, 0.f, 0.f};
  if (sl - L > 0 && col < Dv)
    S = load4<float>(a.state + (((long)a.slot_table[s * a.st_stride] * H + h) * Dv + col) * (long)D + d, D - d, (D & 3) == 0);
  const long base = (long)(t0 / C) + srel;
  const float dc = CHAN ? 0.f : expf(a.log_decay[h] * (float)C);
  for (int c0 = 0; c0 < nch; c0 += 4) {
    f32x4 z[4], dd[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const long id = (base + c0 + u) * H + h;
      z[u] = f32x4{0.f, 0.f, 0.f, 0.f};
      dd[u] = f32x4{dc, dc, dc, dc};
      if (c0 + u < nch - 1) {
        z[u] = *reinterpret_cast<const f32x4*>(a.chunk_state + (id * per + i) * 4);
        if (CHAN) dd[u] = *reinterpret_cast<const f32x4*>(a.chunk_decay + id * DP + d);
      }
    }
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      if (c0 + u < nch) {
        *reinterpret_cast<f32x4*>(a.chunk_state + (((base + c0 + u) * H + h) * per + i) * 4) = S;
        S = S * dd[u] + z[u];
      }
    }
  }
}

static int lin_dt(int D) { return D <= 32 ? 2 : D <= 64 ? 4 : D <= 128 ? 8 : 16; }

// floats of scratch the chunk kernels need for T tokens of S sequences (chunks of C tokens): states, then decays
VDA_EXPORT long vda_linear_attention_scratch(int T, int S, int C, int H, int D, int Dv) {
  const long chunks = (long)T / C + S + 1;
  const int DT = lin_dt(D);
  return chunks * H * ((long)((Dv + 15) / 16) * DT * 256 + DT * 16);
}

VDA_EXPORT int vda_linear_attention_fused(int D, int Dv) {           // can one workgroup hold all of a head's columns?
  return Dv <= (lin_dt(D) <= 8 ? 128 : 64);
}

VDA_EXPORT int vda_linear_attention(
    void* out, long o_stride, float* o_raw, float* scratch, const void* q, long q_stride, const void* k, long k_stride,
    const void* v, long v_stride, const void* z, long z_stride, const float* z_bias, float inv_tau, int decay_exp,
    const float* bonus, const float* log_decay, const void* gate, long g_stride, const float* cos_sin, const long* positions, int rot,
    float q_scale, float k_scale, const float* norm_w, int norm_head, float eps, float* state, const int* qsl, const int* seq_lens,
    const int* slot_table, long st_stride, int T, int S, int seq0, int H, int D, int Dv, int max_q, int C,
    int dtype, hipStream_t st) {
  if (S <= 0 || T <= 0) return 0;
  if (H <= 0 || D < 1 || Dv < 1 || D > 1024 || rot < 0 || rot > D || (rot & 1) || (rot > 0 && (!cos_sin || !positions)) ||
      (!z && !log_decay) || seq0 < 0 || seq0 > S || (bonus && !z) || (norm_head != 0 && norm_head != Dv))
    return -1;
  // chunk-parallel for key widths of up to 256: sequences of more than 16 new tokens, from seq0 on,
  // and only for rows that can be read four values at a time
  const int es = dtype == VDA_F32 ? 16 : 8;
  auto ok4 = [&](const void* p, long stride) { return !p || (((uintptr_t)p % es) == 0 && stride % 4 == 0); };
  const bool vec = D % 4 == 0 && ok4(q, q_stride) && ok4(k, k_stride) && ok4(z, z_stride);
  const bool vec_v = Dv % 4 == 0 && ok4(v, v_stride) && ok4(gate, g_stride) && ok4(out, o_stride) &&
                     !((uintptr_t)norm_w % 16);
  const bool chunked = D <= 256 && max_q > 16 && scratch && seq0 < S && C >= 16 && C % 16 == 0 && vec && vec_v &&
                       rot % 8 == 0 && (!z || rot == 0) && !((uintptr_t)z_bias % 16) && !((uintptr_t)bonus % 16) &&
                       !((uintptr_t)cos_sin % 16);
  const int DT = lin_dt(D);
  const int ET = (DT <= 8 && Dv > 64) ? 2 : 1;
  LinArgs a;
  a.q = q; a.k = k; a.v = v; a.z = z; a.gate = gate;
  a.q_stride = q_stride; a.k_stride = k_stride; a.v_stride = v_stride; a.z_stride = z_stride; a.g_stride = g_stride;
  a.z_bias = z_bias; a.inv_tau = inv_tau; a.decay_exp = decay_exp; a.bonus = bonus; a.norm_head = norm_head; a.log_decay = log_decay; a.cos_sin = cos_sin; a.positions = positions;
  a.rot = rot; a.q_scale = q_scale; a.k_scale = k_scale; a.norm_w = norm_w; a.eps = eps; a.state = state; a.out = out;
  a.o_stride = o_stride; a.qsl = qsl; a.seq_lens = seq_lens; a.slot_table = slot_table; a.st_stride = st_stride;
  a.H = H; a.D = D; a.Dv = Dv; a.seq0 = seq0; a.C = C;
  a.limit = chunked ? 16 : 0x7fffffff;
  a.col_groups = (Dv + 64 * ET - 1) / (64 * ET);
  a.o_raw = a.col_groups > 1 ? o_raw : nullptr;
  if (chunked && a.col_groups > 1 && !o_raw) return -1;
  a.vec = vec;
  const long chunks = chunked ? (long)T / C + (S - seq0) + 1 : 0;
  a.chunk_state = scratch;
  a.chunk_decay = scratch ? scratch + chunks * H * ((long)((Dv + 15) / 16) * DT * 256) : nullptr;
  // few new tokens
  int NR = 1;
  while (16 * NR < D) NR *= 2;
  int tile = max_q < 16 ? max_q : 16;
  auto step_lds = [&](int tl) { return ((size_t)tl * (z ? 3 : 2) * 16 * NR + (size_t)2 * tl * Dv) * 4; };
  while (tile > 1 && step_lds(tile) > 48 * 1024) tile >>= 1;
  if (step_lds(tile) > 60 * 1024) return -2;
  const size_t slds = step_lds(tile);
#define STEP(TT, NN)                                                                                                   \
  do {                                                                                                                 \
    if (bonus) hipLaunchKernelGGL((lin_step_kernel<TT, NN, true, true>), dim3(H, S), dim3(256), slds, st, a, tile);    \
    else if (z) hipLaunchKernelGGL((lin_step_kernel<TT, NN, true, false>), dim3(H, S), dim3(256), slds, st, a, tile);  \
    else hipLaunchKernelGGL((lin_step_kernel<TT, NN, false, false>), dim3(H, S), dim3(256), slds, st, a, tile);        \
  } while (0)
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
  const int nch = (max_q + C - 1) / C;
  const int DP = DT * 16, QP = DP + 4;
  const dim3 grid(nch, S - seq0, H * a.col_groups);
  auto chunk_lds = [&](bool outp) {
    return ((size_t)16 * QP * (1 + (outp ? 1 : 0) + (z ? 1 : 0)) + (size_t)DP * 20 + (size_t)64 * ET * 20 +
            (outp ? (size_t)16 * (64 * ET + 4) : 0) + (z ? DP : 0) + (bonus ? 16 : 0)) * 4;
  };
#define CK(TT, DD, EE, CC, OO, BB)                                                                                       \
  do {                                                                                                                 \
    const size_t lb = chunk_lds(OO);                                                                                   \
    if (lb > 48 * 1024) {                                                                                              \
      hipError_t e_ = hipFuncSetAttribute((const void*)lin_chunk_kernel<TT, DD, EE, CC, OO, BB>,                       \
                                          hipFuncAttributeMaxDynamicSharedMemorySize, (int)lb);                        \
      if (e_ != hipSuccess) return (int)e_;                                                                            \
    }                                                                                                                  \
    hipLaunchKernelGGL((lin_chunk_kernel<TT, DD, EE, CC, OO, BB>), grid, dim3(256), lb, st, a);                        \
  } while (0)
#define CB(TT, DD, EE, OO)                                                                                             \
  do {                                                                                                                 \
    if (OO && bonus) CK(TT, DD, EE, true, OO, OO); /* the bonus concerns the outputs only */                           \
    else if (z) CK(TT, DD, EE, true, OO, false);                                                                       \
    else CK(TT, DD, EE, false, OO, false);                                                                             \
  } while (0)
#define CA(TT, OO)                                                                                                     \
  do {                                                                                                                 \
    if (DT == 2 && ET == 1) CB(TT, 2, 1, OO); else if (DT == 2) CB(TT, 2, 2, OO);                                      \
    else if (DT == 4 && ET == 1) CB(TT, 4, 1, OO); else if (DT == 4) CB(TT, 4, 2, OO);                                 \
    else if (DT == 8 && ET == 1) CB(TT, 8, 1, OO); else if (DT == 8) CB(TT, 8, 2, OO);                                 \
    else CB(TT, 16, 1, OO);                                                                                            \
  } while (0)
#define BYT(OO) do { if (dtype == VDA_BF16) CA(bf16_t, OO); else if (dtype == VDA_F16) CA(f16_t, OO); else CA(float, OO); } while (0)
  if (nch > 1) {
    BYT(false);
    VDA_CHECK_LAUNCH();
    const dim3 gc((((Dv + 15) / 16) * DT * 64 + 255) / 256, S - seq0, H);
    if (z) hipLaunchKernelGGL((lin_carry_kernel<true>), gc, dim3(256), 0, st, a, DT);
    else hipLaunchKernelGGL((lin_carry_kernel<false>), gc, dim3(256), 0, st, a, DT);
    VDA_CHECK_LAUNCH();
  }
  BYT(true);
#undef BYT
#undef CA
#undef CB
#undef CK
  VDA_CHECK_LAUNCH();
  if (a.o_raw) {
    const dim3 ge((unsigned)(((long)max_q * H + 3) / 4), S - seq0);
#define EP(TT) hipLaunchKernelGGL((head_norm_silu_kernel<TT>), ge, dim3(256), 0, st, (TT*)out, o_stride, o_raw,        \
                                  (const TT*)gate, g_stride, norm_w, norm_head, qsl, seq_lens, seq0, a.limit, H, Dv, eps)
    if (dtype == VDA_BF16) EP(bf16_t);
    else if (dtype == VDA_F16) EP(f16_t);
    else EP(float);
#undef EP
    VDA_CHECK_LAUNCH();
  }
  return 0;
}
