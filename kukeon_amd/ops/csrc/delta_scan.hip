// Gated delta rule, the recurrent form. Per head, with unit keys and queries
// k~ = k / sqrt(|k|^2 + 1e-6), q~ = q / sqrt(|q|^2 + 1e-6) * q_scale,
// beta = sigmoid(b) and the decay g = exp(-rate softplus(a + dt_bias)):
//
//   S <- g S ;  u = beta (v - S^T k~) ;  S <- S + k~ u^T ;  o = S^T q~
//
// Both reads of the state can be taken from the OLD one,
//   S^T k~ = g S_old^T k~ ,   o = g S_old^T q~ + (k~ . q~) u ,
// so a token costs one pass over the state and one reduction, and the norms
// never touch the staged rows: 1/|k|, 1/|q| and k.q are per-token scalars.
//
// The columns of S are independent, so a workgroup takes one (sequence, head,
// block of value columns). The state stays in registers for the whole portion:
// the LN lanes of a column own its key rows in interleaved pieces of four
// (row = (4 i + lane) 4 + j, which keeps LDS reads and slot accesses
// contiguous over the lanes), and the partial dot products meet by lane moves
// inside the wave. q, k, v of TT tokens are staged in LDS at a time, rows
// padded with zeros. The slot holds S^T ([H, dv, d]); it is read once at the
// start of the portion (zeros at position 0, whatever the slot held) and
// written once at its end. Tokens are visited in order, so a position's result
// does not depend on how the sequence was cut. Everything is fp32.
#include "elem.h"

namespace kukeon {

template <int CTRL>
DEV_INLINE float dpp_add(float v) {
  const int m = __builtin_amdgcn_update_dpp(
      0, __builtin_bit_cast(int, v), CTRL, 0xf, 0xf, true);
  return v + __builtin_bit_cast(float, m);
}
// sum over LN (<= 16) neighbouring lanes, the result in all of them: swap in
// pairs, swap pairs, then mirror halves of 8 and of 16
template <int LN>
DEV_INLINE float lanes_sum(float v) {
  if (LN > 1) v = dpp_add<0xB1>(v);      // quad_perm [1,0,3,2]
  if (LN > 2) v = dpp_add<0x4E>(v);      // quad_perm [2,3,0,1]
  if (LN > 4) v = dpp_add<0x141>(v);     // row_half_mirror
  if (LN > 8) v = dpp_add<0x140>(v);     // row_mirror
  return v;
}

template <typename T, int LN, int NR>
__global__ __launch_bounds__(256) void delta_scan_kernel(
    float* __restrict__ y, const T* __restrict__ qkv, long ldq, long q_col,
    long k_col, long v_col, const T* __restrict__ ba, long ldb, long b_col,
    long a_col, const float* __restrict__ rate,
    const float* __restrict__ dt_bias, float q_scale, float* __restrict__ state,
    const int* __restrict__ positions, const int* __restrict__ cu_rows,
    const int* __restrict__ state_slots, int H, int G, int d, int dv) {
  constexpr int DP = LN * NR;            // padded key row
  constexpr int NC = 256 / LN;           // value columns of the workgroup
  constexpr int TT = DP > 256 ? 8 : 16;  // tokens staged at a time
  __shared__ __align__(16) float sQ[TT * DP];
  __shared__ __align__(16) float sK[TT * DP];
  __shared__ float sV[TT * NC];
  __shared__ float sG[TT], sB[TT], sRk[TT], sRq[TT], sKQ[TT];
  const int s = blockIdx.x;
  const int h = blockIdx.y;
  const int c0 = blockIdx.z * NC;
  const long row0 = cu_rows[s];
  const int n = cu_rows[s + 1] - (int)row0;
  if (n <= 0) return;
  const int p0 = positions[row0];
  const int tid = threadIdx.x;
  const int nc = min(NC, dv - c0);
  const int inner = H * dv;
  if (p0 < 0) {                          // inactive sequence: zeros out
    for (int i = tid; i < n * nc; i += 256)
      y[(row0 + i / nc) * (long)inner + h * dv + c0 + i % nc] = 0.f;
    return;
  }
  const int kh = h / (H / G);
  const T* qp = qkv + q_col + (long)kh * d;
  const T* kp = qkv + k_col + (long)kh * d;
  const T* vp = qkv + v_col + (long)h * dv + c0;
  const float rate_h = rate[h], bias_h = dt_bias[h];
  const int e = tid / LN;
  const int l = tid - e * LN;
  const bool live = e < nc;
  // A short portion's few inputs are fetched ahead of the state: loads
  // complete in issue order, and what comes after the state waits for it.
  const bool pre = n * DP <= 256 && n * nc <= 256 && n <= TT;
  float pq = 0.f, pk = 0.f, pv = 0.f, pa = 0.f, pb = 0.f;
  if (pre) {
    const int t = tid / DP, dd = tid - t * DP;
    if (t < n && dd < d) {
      pq = ldf(qp + (row0 + t) * ldq + dd);
      pk = ldf(kp + (row0 + t) * ldq + dd);
    }
    if (tid < n * nc) pv = ldf(vp + (row0 + tid / nc) * ldq + tid % nc);
    if (tid < n) {
      pa = ldf(ba + (row0 + tid) * ldb + a_col + h);
      pb = ldf(ba + (row0 + tid) * ldb + b_col + h);
    }
  }
  float* st = state + (((long)state_slots[s] * H + h) * dv + c0 +
                       (live ? e : 0)) * (long)d;
  const bool vec4 = (d & 3) == 0;
  float S[NR];
#pragma unroll
  for (int i = 0; i < NR / 4; ++i) {
    const int dd = (i * LN + l) * 4;
    float4 x = float4{0.f, 0.f, 0.f, 0.f};
    if (live && p0 > 0) {
      if (vec4) {
        if (dd < d) x = *reinterpret_cast<const float4*>(st + dd);
      } else {
        if (dd + 0 < d) x.x = st[dd + 0];
        if (dd + 1 < d) x.y = st[dd + 1];
        if (dd + 2 < d) x.z = st[dd + 2];
        if (dd + 3 < d) x.w = st[dd + 3];
      }
    }
    S[4 * i] = x.x; S[4 * i + 1] = x.y; S[4 * i + 2] = x.z; S[4 * i + 3] = x.w;
  }
  for (int t0 = 0; t0 < n; t0 += TT) {
    const int nt = min(TT, n - t0);
    const long r0 = row0 + t0;
    __syncthreads();
    for (int i = tid; i < nt * DP; i += 256) {
      const int t = i / DP, dd = i - t * DP;
      float qv = 0.f, kv = 0.f;
      if (pre) {
        qv = pq; kv = pk;
      } else if (dd < d) {
        qv = ldf(qp + (r0 + t) * ldq + dd);
        kv = ldf(kp + (r0 + t) * ldq + dd);
      }
      sQ[i] = qv; sK[i] = kv;
    }
    for (int i = tid; i < nt * nc; i += 256) {
      const int t = i / nc, ee = i - t * nc;
      sV[t * NC + ee] = pre ? pv : ldf(vp + (r0 + t) * ldq + ee);
    }
    if (tid < nt) {
      const float a = (pre ? pa : ldf(ba + (r0 + tid) * ldb + a_col + h)) +
                      bias_h;
      const float b = pre ? pb : ldf(ba + (r0 + tid) * ldb + b_col + h);
      const float sp = a > 20.f ? a : log1pf(expf(a));
      sG[tid] = expf(-rate_h * sp);
      sB[tid] = 1.0f / (1.0f + expf(-b));
    }
    __syncthreads();
    // 16 lanes per token share out the key row's three sums
    for (int i = tid; i < nt * 16; i += 256) {
      const int t = i >> 4, part = i & 15;
      float qq = 0.f, kk = 0.f, kq = 0.f;
      for (int dd = part; dd < d; dd += 16) {
        const float a = sQ[t * DP + dd], b = sK[t * DP + dd];
        qq = fmaf(a, a, qq);
        kk = fmaf(b, b, kk);
        kq = fmaf(a, b, kq);
      }
      qq = lanes_sum<16>(qq);
      kk = lanes_sum<16>(kk);
      kq = lanes_sum<16>(kq);
      if (part == 0) {
        const float rk = 1.0f / sqrtf(kk + 1e-6f);
        const float rq = q_scale / sqrtf(qq + 1e-6f);
        sRk[t] = rk;
        sRq[t] = rq;
        sKQ[t] = kq * rk * rq;
      }
    }
    __syncthreads();
    if (live) {
      for (int t = 0; t < nt; ++t) {
        const float4* kt = reinterpret_cast<const float4*>(sK + t * DP) + l;
        const float4* qt = reinterpret_cast<const float4*>(sQ + t * DP) + l;
        float4 k4[NR / 4];
        float dk[4] = {0.f, 0.f, 0.f, 0.f}, dq[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int i = 0; i < NR / 4; ++i) {
          k4[i] = kt[i * LN];
          const float4 q4 = qt[i * LN];
          dk[0] = fmaf(S[4 * i + 0], k4[i].x, dk[0]);
          dk[1] = fmaf(S[4 * i + 1], k4[i].y, dk[1]);
          dk[2] = fmaf(S[4 * i + 2], k4[i].z, dk[2]);
          dk[3] = fmaf(S[4 * i + 3], k4[i].w, dk[3]);
          dq[0] = fmaf(S[4 * i + 0], q4.x, dq[0]);
          dq[1] = fmaf(S[4 * i + 1], q4.y, dq[1]);
          dq[2] = fmaf(S[4 * i + 2], q4.z, dq[2]);
          dq[3] = fmaf(S[4 * i + 3], q4.w, dq[3]);
        }
        const float g = sG[t], rk = sRk[t];
        const float sk = lanes_sum<LN>((dk[0] + dk[1]) + (dk[2] + dk[3]));
        const float sq = lanes_sum<LN>((dq[0] + dq[1]) + (dq[2] + dq[3]));
        const float u = sB[t] * (sV[t * NC + e] - g * rk * sk);
        const float ku = rk * u;
#pragma unroll
        for (int i = 0; i < NR / 4; ++i) {
          S[4 * i + 0] = fmaf(k4[i].x, ku, g * S[4 * i + 0]);
          S[4 * i + 1] = fmaf(k4[i].y, ku, g * S[4 * i + 1]);
          S[4 * i + 2] = fmaf(k4[i].z, ku, g * S[4 * i + 2]);
          S[4 * i + 3] = fmaf(k4[i].w, ku, g * S[4 * i + 3]);
        }
        if (l == 0)
          y[(r0 + t) * (long)inner + h * dv + c0 + e] =
              fmaf(sKQ[t], u, g * sRq[t] * sq);
      }
    }
  }
  if (live) {
#pragma unroll
    for (int i = 0; i < NR / 4; ++i) {
      const int dd = (i * LN + l) * 4;
      if (vec4) {
        if (dd < d)
          *reinterpret_cast<float4*>(st + dd) =
              float4{S[4 * i], S[4 * i + 1], S[4 * i + 2], S[4 * i + 3]};
      } else {
#pragma unroll
        for (int j = 0; j < 4; ++j)
          if (dd + j < d) st[dd + j] = S[4 * i + j];
      }
    }
  }
}

// y [T, H*dv] fp32; qkv [T, ld] (stride(1) == 1): q and k at G*d columns from
// q_col / k_col, v at H*dv columns from v_col; ba [T, ld]: H columns of b and
// of a; rate, dt_bias [H] fp32; state [slots, H, dv, d] fp32.
void delta_scan(torch::Tensor y, torch::Tensor qkv, int64_t q_col,
                int64_t k_col, int64_t v_col, torch::Tensor ba, int64_t b_col,
                int64_t a_col, torch::Tensor rate, torch::Tensor dt_bias,
                double q_scale, torch::Tensor state, torch::Tensor positions,
                torch::Tensor cu_rows, torch::Tensor state_slots, int64_t H,
                int64_t G, int64_t d, int64_t dv) {
  check_act(qkv, "qkv"); check_act(ba, "ba");
  check_f32(y, "y"); check_f32(rate, "rate"); check_f32(dt_bias, "dt_bias");
  check_f32(state, "state");
  check_i32(positions, "positions"); check_i32(cu_rows, "cu_rows");
  check_i32(state_slots, "state_slots");
  TORCH_CHECK(H >= 1 && G >= 1 && H % G == 0 && d >= 1 && dv >= 1);
  const long rows = qkv.size(0);
  TORCH_CHECK(qkv.dim() == 2 && qkv.stride(1) == 1 && ba.dim() == 2 &&
              ba.stride(1) == 1 && ba.size(0) == rows &&
              ba.scalar_type() == qkv.scalar_type());
  TORCH_CHECK(q_col >= 0 && q_col + G * d <= qkv.size(1) && k_col >= 0 &&
              k_col + G * d <= qkv.size(1) && v_col >= 0 &&
              v_col + H * dv <= qkv.size(1));
  TORCH_CHECK(b_col >= 0 && b_col + H <= ba.size(1) && a_col >= 0 &&
              a_col + H <= ba.size(1));
  TORCH_CHECK(y.dim() == 2 && y.size(0) == rows && y.size(1) == H * dv);
  TORCH_CHECK(rate.numel() == H && dt_bias.numel() == H);
  TORCH_CHECK(state.dim() == 4 && state.size(1) == H && state.size(2) == dv &&
              state.size(3) == d);
  TORCH_CHECK(positions.numel() == rows);
  const long nseq = cu_rows.numel() - 1;
  TORCH_CHECK(nseq >= 0 && state_slots.numel() >= nseq);
  if (rows == 0 || nseq == 0) return;
  TORCH_CHECK(d <= 512, "delta_scan: key rows of more than 512 entries");
  // steps of one token per sequence are bound by the state's bytes: many
  // lanes per column, few rows each; portions by the work per token
  const bool step = rows == nseq;
  auto stream = c10::hip::getCurrentHIPStream().stream();
#define KK_LAUNCH(LN_, NR_)                                                   \
  {                                                                           \
    dim3 grid((unsigned)nseq, (unsigned)H,                                    \
              (unsigned)((dv + 256 / LN_ - 1) / (256 / LN_)));                \
    delta_scan_kernel<T, LN_, NR_><<<grid, 256, 0, stream>>>(                 \
        y.data_ptr<float>(), reinterpret_cast<const T*>(qkv.data_ptr()),      \
        (long)qkv.stride(0), (long)q_col, (long)k_col, (long)v_col,           \
        reinterpret_cast<const T*>(ba.data_ptr()), (long)ba.stride(0),        \
        (long)b_col, (long)a_col, rate.data_ptr<float>(),                     \
        dt_bias.data_ptr<float>(), (float)q_scale, state.data_ptr<float>(),   \
        positions.data_ptr<int>(), cu_rows.data_ptr<int>(),                   \
        state_slots.data_ptr<int>(), (int)H, (int)G, (int)d, (int)dv);        \
  }
  KK_DISPATCH_ACT(qkv, {
    if (d <= 32) KK_LAUNCH(8, 4)
    else if (d <= 64) { if (step) KK_LAUNCH(16, 4) else KK_LAUNCH(4, 16) }
    else if (d <= 128) { if (step) KK_LAUNCH(16, 8) else KK_LAUNCH(4, 32) }
    else if (d <= 256) { if (step) KK_LAUNCH(16, 16) else KK_LAUNCH(8, 32) }
    else KK_LAUNCH(16, 32)
  });
#undef KK_LAUNCH
  HIP_CHECK_KERNEL();
}

}  // namespace kukeon
