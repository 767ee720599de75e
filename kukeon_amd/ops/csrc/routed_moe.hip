// Router side of a mixture of experts chosen by learned logits:
//   router_topk            per row, the `top` largest logits (ties: the lower
//                          index) and the softmax over just those, fp32
//   router_select          scores = softmax over ALL logits; the experts form
//                          equal runs of neighbours of which only the best
//                          few (by their largest score) can be chosen; the
//                          chosen scores are divided by their sum and scaled
//   router_sigmoid         scores = sigmoid of every logit by itself; the `top`
//                          largest, as they are, times a scale
//   router_corrected       scores = sigmoid of every logit; the choice goes by
//                          score plus a learned correction per expert, within
//                          the best runs of neighbours (by the sum of a run's
//                          largest few choice scores); the weights are the
//                          scores without it, divided by their sum if asked
//   combine_rows_weighted  out[t] = sum_k w[t, k] * in[inv[t, k]], the k-th
//                          term added k-th, fp32 sums
// The expert GEMMs themselves are vendor GEMMs over gathered rows.
#include "elem.h"

namespace kukeon {

// One thread per row. The k-th pick is the largest (value, -index) pair
// below the previous pick, so no list of taken experts is kept; a NaN logit
// counts as -inf, which keeps every index in range.
__global__ __launch_bounds__(256) void router_topk_kernel(
    int* __restrict__ idx, float* __restrict__ wts,
    const float* __restrict__ logits, long rows, int E, int top,
    long dense_rows) {
  const long t = (long)blockIdx.x * blockDim.x + threadIdx.x;
  if (t >= rows) return;
  const float* z = logits + t * (long)E;
  float pv = INFINITY;
  int pe = -1;
  float vmax = 0.f, sum = 0.f;
  for (int k = 0; k < top; ++k) {
    float bv = -INFINITY;
    int be = -1;
    for (int e = 0; e < E; ++e) {
      float v = z[e];
      v = v == v ? v : -INFINITY;
      const bool below = v < pv || (v == pv && e > pe);
      const bool better = be < 0 || v > bv;
      if (below && better) { bv = v; be = e; }
    }
    pv = bv;
    pe = be;
    if (k == 0) vmax = bv;
    const float w = expf(bv - vmax);
    wts[t * top + k] = w;
    sum += w;
    idx[t * top + k] = dense_rows > 0 ? (int)(be * dense_rows + t) : be;
  }
  const float inv = 1.0f / sum;
  for (int k = 0; k < top; ++k) wts[t * top + k] *= inv;
}

// idx [T, top] int32, wts [T, top] fp32, logits [T, E] fp32. With
// dense_rows = T the index written is expert * T + row.
void router_topk(torch::Tensor idx, torch::Tensor wts, torch::Tensor logits,
                 int64_t top, int64_t dense_rows) {
  check_i32(idx, "idx"); check_f32(wts, "wts"); check_f32(logits, "logits");
  TORCH_CHECK(logits.dim() == 2);
  const long rows = logits.size(0);
  const int E = (int)logits.size(1);
  TORCH_CHECK(top >= 1 && top <= E);
  TORCH_CHECK(idx.numel() == rows * top && wts.numel() == rows * top);
  TORCH_CHECK(dense_rows == 0 || dense_rows == rows);
  TORCH_CHECK((long)E * rows < (1L << 31));
  if (rows == 0) return;
  auto stream = c10::hip::getCurrentHIPStream().stream();
  router_topk_kernel<<<dim3((unsigned)((rows + 255) / 256)), 256, 0, stream>>>(
      idx.data_ptr<int>(), wts.data_ptr<float>(), logits.data_ptr<float>(),
      rows, E, (int)top, (long)dense_rows);
  HIP_CHECK_KERNEL();
}

// One thread per row. A softmax keeps the order of the logits, so runs and
// experts are ranked by logit; every pick is the largest (value, -index) pair
// below the previous pick. A NaN logit counts as -inf.
__global__ __launch_bounds__(256) void router_select_kernel(
    int* __restrict__ idx, float* __restrict__ wts, long ldi, long ldw,
    const float* __restrict__ logits, long ldz, long rows, int E, int top,
    int groups, int keep, float scale, long dense_rows) {
  const long t = (long)blockIdx.x * blockDim.x + threadIdx.x;
  if (t >= rows) return;
  const float* z = logits + t * ldz;
  float vmax = -INFINITY;
  for (int e = 0; e < E; ++e) {
    const float v = z[e];
    if (v == v) vmax = fmaxf(vmax, v);
  }
  if (vmax == -INFINITY) vmax = 0.f;         // a row of NaN: finite weights
  float sum = 0.f;
  for (int e = 0; e < E; ++e) {
    const float v = z[e];
    if (v == v) sum += expf(v - vmax);
  }
  unsigned long long allowed = ~0ull;        // one bit per run
  const int per = groups > 0 ? E / groups : E;
  if (groups > 0) {
    allowed = 0ull;
    float pv = INFINITY;
    int pg = -1;
    for (int k = 0; k < keep; ++k) {
      float bv = -INFINITY;
      int bg = -1;
      for (int g = 0; g < groups; ++g) {
        float gv = -INFINITY;
        for (int e = g * per; e < (g + 1) * per; ++e) {
          const float v = z[e];
          if (v == v) gv = fmaxf(gv, v);
        }
        const bool below = gv < pv || (gv == pv && g > pg);
        const bool better = bg < 0 || gv > bv;
        if (below && better) { bv = gv; bg = g; }
      }
      pv = bv;
      pg = bg;
      allowed |= 1ull << bg;
    }
  }
  float pv = INFINITY;
  int pe = -1;
  float wsum = 0.f;
  for (int k = 0; k < top; ++k) {
    float bv = -INFINITY;
    int be = -1;
    for (int e = 0; e < E; ++e) {
      if (groups > 0 && !((allowed >> (e / per)) & 1ull)) continue;
      float v = z[e];
      v = v == v ? v : -INFINITY;
      const bool below = v < pv || (v == pv && e > pe);
      const bool better = be < 0 || v > bv;
      if (below && better) { bv = v; be = e; }
    }
    pv = bv;
    pe = be;
    const float w = expf(bv - vmax) / sum;
    wts[t * ldw + k] = w;
    wsum += w;
    idx[t * ldi + k] = dense_rows > 0 ? (int)(be * dense_rows + t) : be;
  }
  const float f = scale / (wsum + 1e-20f);
  for (int k = 0; k < top; ++k) wts[t * ldw + k] *= f;
}

// idx [T, >= top] int32, wts [T, >= top] fp32 (rows may be wider than top:
// the other columns are left alone), logits [T, E] fp32 (any row stride: the
// first E columns of a wider product).
void router_select(torch::Tensor idx, torch::Tensor wts, torch::Tensor logits,
                   int64_t top, int64_t groups, int64_t keep, double scale,
                   int64_t dense_rows) {
  TORCH_CHECK(logits.is_cuda() && logits.scalar_type() == torch::kFloat32 &&
              logits.dim() == 2 && logits.stride(1) == 1,
              "logits must be fp32 rows");
  TORCH_CHECK(idx.is_cuda() && idx.scalar_type() == torch::kInt32 &&
              wts.is_cuda() && wts.scalar_type() == torch::kFloat32);
  TORCH_CHECK(idx.dim() == 2 && wts.dim() == 2);
  const long rows = logits.size(0);
  const int E = (int)logits.size(1);
  TORCH_CHECK(top >= 1 && top <= E);
  TORCH_CHECK(idx.size(0) == rows && wts.size(0) == rows &&
              idx.size(1) >= top && wts.size(1) >= top &&
              idx.stride(1) == 1 && wts.stride(1) == 1);
  TORCH_CHECK(groups >= 0 && groups <= 64);
  if (groups > 0)
    TORCH_CHECK(E % groups == 0 && keep >= 1 && keep <= groups &&
                top <= keep * (E / groups));
  TORCH_CHECK(dense_rows == 0 || dense_rows == rows);
  TORCH_CHECK((long)E * rows < (1L << 31));
  if (rows == 0) return;
  auto stream = c10::hip::getCurrentHIPStream().stream();
  router_select_kernel<<<dim3((unsigned)((rows + 255) / 256)), 256, 0,
                         stream>>>(
      idx.data_ptr<int>(), wts.data_ptr<float>(), (long)idx.stride(0),
      (long)wts.stride(0), logits.data_ptr<float>(), (long)logits.stride(0),
      rows, E, (int)top, (int)groups, (int)keep, (float)scale,
      (long)dense_rows);
  HIP_CHECK_KERNEL();
}

// One thread per row; a sigmoid keeps the order of the logits.
__global__ __launch_bounds__(64) void router_sigmoid_kernel(
    int* __restrict__ idx, float* __restrict__ wts, long ldi, long ldw,
    const float* __restrict__ logits, long ldz, long rows, int E, int top,
    float scale) {
  const long t = (long)blockIdx.x * blockDim.x + threadIdx.x;
  if (t >= rows) return;
  const float* z = logits + t * ldz;
  float pv = INFINITY;
  int pe = -1;
  for (int k = 0; k < top; ++k) {
    float bv = -INFINITY;
    int be = -1;
    for (int e = 0; e < E; ++e) {
      float v = z[e];
      v = v == v ? v : -INFINITY;
      const bool below = v < pv || (v == pv && e > pe);
      const bool better = be < 0 || v > bv;
      if (below && better) { bv = v; be = e; }
    }
    pv = bv;
    pe = be;
    wts[t * ldw + k] = scale / (1.0f + expf(-bv));
    idx[t * ldi + k] = be;
  }
}

// idx [T, >= top] int32, wts [T, >= top] fp32, logits [T, E] fp32 (row strides
// free).
void router_sigmoid(torch::Tensor idx, torch::Tensor wts, torch::Tensor logits,
                    int64_t top, double scale) {
  TORCH_CHECK(logits.is_cuda() && logits.scalar_type() == torch::kFloat32 &&
              logits.dim() == 2 && logits.stride(1) == 1,
              "logits must be fp32 rows");
  TORCH_CHECK(idx.is_cuda() && idx.scalar_type() == torch::kInt32 &&
              wts.is_cuda() && wts.scalar_type() == torch::kFloat32);
  TORCH_CHECK(idx.dim() == 2 && wts.dim() == 2);
  const long rows = logits.size(0);
  const int E = (int)logits.size(1);
  TORCH_CHECK(top >= 1 && top <= E);
  TORCH_CHECK(idx.size(0) == rows && wts.size(0) == rows &&
              idx.size(1) >= top && wts.size(1) >= top &&
              idx.stride(1) == 1 && wts.stride(1) == 1);
  if (rows == 0) return;
  auto stream = c10::hip::getCurrentHIPStream().stream();
  router_sigmoid_kernel<<<dim3((unsigned)((rows + 63) / 64)), 64, 0, stream>>>(
      idx.data_ptr<int>(), wts.data_ptr<float>(), (long)idx.stride(0),
      (long)wts.stride(0), logits.data_ptr<float>(), (long)logits.stride(0),
      rows, E, (int)top, (float)scale);
  HIP_CHECK_KERNEL();
}

// The largest (value, -index) pair of a wave; every lane gets the index.
DEV_INLINE int wave_argmax(float v, int i) {
#pragma unroll
  for (int off = 32; off > 0; off >>= 1) {
    const float ov = __shfl_xor(v, off, WAVE);
    const int oi = __shfl_xor(i, off, WAVE);
    if (ov > v || (ov == v && oi < i)) { v = ov; i = oi; }
  }
  return i;
}

// Score and choice score of a logit: a NaN counts as a score of 0 and the lowest
// choice score, and no choice score is -inf, which marks what cannot be chosen.
DEV_INLINE void corrected_score(float z, float corr, float& s, float& c) {
  s = 1.0f / (1.0f + expf(-z));
  c = s + corr;
  c = c == c ? fmaxf(c, -3.0e38f) : -3.0e38f;
  s = s == s ? s : 0.f;
}

// Up to 64 experts: one wave per row, lane = expert, everything by lane moves.
// An expert's rank is the number of experts ahead of it (larger, or equal with
// a lower index); ranks below `top` are the choice, in order.
__global__ __launch_bounds__(256) void router_corrected_wave_kernel(
    int* __restrict__ idx, float* __restrict__ wts, long ldi, long ldw,
    const float* __restrict__ logits, long ldz,
    const float* __restrict__ correction, long rows, int E, int top, int groups,
    int keep, int best, float scale, int renorm) {
  const long t = (long)blockIdx.x * 4 + threadIdx.x / WAVE;
  if (t >= rows) return;                 // a whole wave
  const int e = threadIdx.x & (WAVE - 1);
  float s = 0.f, c = -INFINITY;
  if (e < E)
    corrected_score(logits[t * ldz + e], correction ? correction[e] : 0.f, s,
                    c);
  if (groups > 0) {
    const int per = E / groups;
    const int g = e / per;               // lanes past E are in no run
    float a = -INFINITY, b = -INFINITY;  // the run's two largest
    for (int i = 0; i < per; ++i) {
      const float v = __shfl(c, min(g * per + i, WAVE - 1), WAVE);
      b = fmaxf(b, fminf(a, v));
      a = fmaxf(a, v);
    }
    const float gv = fmaxf(best > 1 && per > 1 ? a + b : a, -3.0e38f);
    int rank = 0;
    for (int o = 0; o < groups; ++o) {
      const float v = __shfl(gv, o * per, WAVE);
      rank += v > gv || (v == gv && o < g);
    }
    if (rank >= keep || e >= E) c = -INFINITY;
  }
  int rank = 0;
  for (int o = 0; o < E; ++o) {
    const float v = __shfl(c, o, WAVE);
    rank += v > c || (v == c && o < e);
  }
  const bool chosen = e < E && rank < top;
  const float sum = wave_sum(chosen ? s : 0.f);
  if (chosen) {
    idx[t * ldi + rank] = e;
    wts[t * ldw + rank] = s * (renorm ? scale / (sum + 1e-20f) : scale);
  }
}

// More experts: one wave per row, the experts in turns over the lanes. In LDS:
// scores s [E], choice scores c [E], run scores [groups].
__global__ __launch_bounds__(64) void router_corrected_kernel(
    int* __restrict__ idx, float* __restrict__ wts, long ldi, long ldw,
    const float* __restrict__ logits, long ldz,
    const float* __restrict__ correction, int E, int top, int groups, int keep,
    int best, float scale, int renorm) {
  extern __shared__ float sm[];
  float* s = sm;
  float* c = s + E;
  float* gs = c + E;
  const long t = blockIdx.x;
  const int lane = threadIdx.x;
  const float* z = logits + t * ldz;
  for (int e = lane; e < E; e += WAVE) {
    float sc, ch;
    corrected_score(z[e], correction ? correction[e] : 0.f, sc, ch);
    s[e] = sc;
    c[e] = ch;
  }
  __syncthreads();
  if (groups > 0) {
    const int per = E / groups;
    for (int g = lane; g < groups; g += WAVE) {
      float a = -INFINITY, b = -INFINITY;       // the two largest
      for (int e = g * per; e < (g + 1) * per; ++e) {
        const float v = c[e];
        b = fmaxf(b, fminf(a, v));
        a = fmaxf(a, v);
      }
      gs[g] = fmaxf(best > 1 && per > 1 ? a + b : a, -3.0e38f);
    }
    __syncthreads();
    for (int k = 0; k < keep; ++k) {
      float v = -INFINITY;
      int i = groups;
      for (int g = lane; g < groups; g += WAVE)
        if (gs[g] > v) { v = gs[g]; i = g; }
      i = min(wave_argmax(v, i), groups - 1);
      __syncthreads();
      if (lane == 0) gs[i] = -INFINITY;         // taken
      __syncthreads();
    }
    for (int e = lane; e < E; e += WAVE)
      if (gs[e / per] != -INFINITY) c[e] = -INFINITY;
    __syncthreads();
  }
  float sum = 0.f;
  for (int k = 0; k < top; ++k) {
    float v = -INFINITY;
    int i = E;
    for (int e = lane; e < E; e += WAVE)
      if (c[e] > v) { v = c[e]; i = e; }
    i = min(wave_argmax(v, i), E - 1);
    sum += s[i];
    if (lane == 0) idx[t * ldi + k] = i;
    if (lane == (k & (WAVE - 1))) wts[t * ldw + k] = s[i];
    __syncthreads();
    if (lane == 0) c[i] = -INFINITY;
    __syncthreads();
  }
  const float f = renorm ? scale / (sum + 1e-20f) : scale;
  // lane k & 63 wrote weight k and reads it back
  for (int k = lane; k < top; k += WAVE) wts[t * ldw + k] *= f;
}

// idx [T, >= top] int32, wts [T, >= top] fp32, logits [T, E] fp32 (row strides
// free); correction [E] fp32 or empty; groups 0: every expert can be chosen;
// best: how many of a run's largest choice scores make its own (1 or 2).
void router_corrected(torch::Tensor idx, torch::Tensor wts,
                      torch::Tensor logits, torch::Tensor correction,
                      int64_t top, int64_t groups, int64_t keep, int64_t best,
                      double scale, bool renorm) {
  TORCH_CHECK(logits.is_cuda() && logits.scalar_type() == torch::kFloat32 &&
              logits.dim() == 2 && logits.stride(1) == 1,
              "logits must be fp32 rows");
  TORCH_CHECK(idx.is_cuda() && idx.scalar_type() == torch::kInt32 &&
              wts.is_cuda() && wts.scalar_type() == torch::kFloat32);
  TORCH_CHECK(idx.dim() == 2 && wts.dim() == 2);
  const long rows = logits.size(0);
  const int E = (int)logits.size(1);
  TORCH_CHECK(top >= 1 && top <= E && (best == 1 || best == 2));
  TORCH_CHECK(idx.size(0) == rows && wts.size(0) == rows &&
              idx.size(1) >= top && wts.size(1) >= top &&
              idx.stride(1) == 1 && wts.stride(1) == 1);
  TORCH_CHECK(groups >= 0 && groups <= E);
  if (groups > 0)
    TORCH_CHECK(E % groups == 0 && keep >= 1 && keep <= groups &&
                top <= keep * (E / groups));
  const bool corr = correction.numel() > 0;
  if (corr) {
    check_f32(correction, "correction");
    TORCH_CHECK(correction.numel() == E);
  }
  const size_t lds = (size_t)(2 * E + groups) * sizeof(float);
  TORCH_CHECK(lds <= 60 * 1024, "router_corrected: too many experts");
  if (rows == 0) return;
  auto stream = c10::hip::getCurrentHIPStream().stream();
  if (E <= WAVE) {
    router_corrected_wave_kernel<<<dim3((unsigned)((rows + 3) / 4)), 256, 0,
                                   stream>>>(
        idx.data_ptr<int>(), wts.data_ptr<float>(), (long)idx.stride(0),
        (long)wts.stride(0), logits.data_ptr<float>(), (long)logits.stride(0),
        corr ? correction.data_ptr<float>() : nullptr, rows, E, (int)top,
        (int)groups, (int)keep, (int)best, (float)scale, (int)renorm);
    HIP_CHECK_KERNEL();
    return;
  }
  router_corrected_kernel<<<dim3((unsigned)rows), 64, lds, stream>>>(
      idx.data_ptr<int>(), wts.data_ptr<float>(), (long)idx.stride(0),
      (long)wts.stride(0), logits.data_ptr<float>(), (long)logits.stride(0),
      corr ? correction.data_ptr<float>() : nullptr, E, (int)top, (int)groups,
      (int)keep, (int)best, (float)scale, (int)renorm);
  HIP_CHECK_KERNEL();
}

template <typename T>
__global__ __launch_bounds__(256) void combine_rows_weighted_kernel(
    T* __restrict__ out, const T* __restrict__ in, const int* __restrict__ inv,
    const float* __restrict__ wts, int W, int top) {
  const long t = blockIdx.x;
  if (W % 8 == 0 && aligned16(in) && aligned16(out)) {
    for (int i = threadIdx.x * 8; i < W; i += blockDim.x * 8) {
      float acc[8];
#pragma unroll
      for (int j = 0; j < 8; ++j) acc[j] = 0.f;
      for (int k = 0; k < top; ++k) {
        float v[8];
        ld8(in + (long)inv[t * top + k] * W + i, v);
        const float w = wts[t * top + k];
#pragma unroll
        for (int j = 0; j < 8; ++j) acc[j] = fmaf(w, v[j], acc[j]);
      }
      st8(out + t * (long)W + i, acc);
    }
    return;
  }
  for (int i = threadIdx.x; i < W; i += blockDim.x) {
    float acc = 0.f;
    for (int k = 0; k < top; ++k)
      acc = fmaf(wts[t * top + k], ldf(in + (long)inv[t * top + k] * W + i),
                 acc);
    stf(out + t * (long)W + i, acc);
  }
}

// out [T, W]; in [n, W]; inv [T, top] rows of `in`; wts [T, top] fp32.
void combine_rows_weighted(torch::Tensor out, torch::Tensor in,
                           torch::Tensor inv, torch::Tensor wts) {
  check_act(out, "out"); check_act(in, "in"); check_i32(inv, "inv");
  check_f32(wts, "wts");
  TORCH_CHECK(out.dim() == 2 && in.dim() == 2 && out.is_contiguous() &&
              in.is_contiguous() && out.size(1) == in.size(1) &&
              out.scalar_type() == in.scalar_type());
  TORCH_CHECK(inv.dim() == 2 && inv.size(0) == out.size(0) &&
              wts.dim() == 2 && wts.size(0) == inv.size(0) &&
              wts.size(1) == inv.size(1));
  const long n = out.size(0);
  if (n == 0) return;
  auto stream = c10::hip::getCurrentHIPStream().stream();
  KK_DISPATCH_ACT(out, {
    combine_rows_weighted_kernel<T><<<dim3((unsigned)n), 256, 0, stream>>>(
        reinterpret_cast<T*>(out.data_ptr()),
        reinterpret_cast<const T*>(in.data_ptr()), inv.data_ptr<int>(),
        wts.data_ptr<float>(), (int)out.size(1), (int)inv.size(1));
  });
  HIP_CHECK_KERNEL();
}

}  // namespace kukeon
