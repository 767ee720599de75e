// Residual step of a stack that norms AFTER the sum, in one pass over a row
// of the fp32 stream:
//
//   x <- norm(alpha * x + scale * y) * w
//
// norm is the RMS norm in `groups` equal runs of neighbouring entries (one
// run: the plain RMS norm), scale a per-entry factor of the sublayer's output
// y. The same launch can prepare what reads x next:
//   NEXT 0  nothing (a prompt portion: the convolution of the next input
//           needs the rows before this one)
//   NEXT 1  h = x + conv(x), the next sublayer's causally convolved input, for
//           steps in which every sequence brings one row: the taps before it
//           come from the state slot, which is shifted here
//   NEXT 2  h = norm(x) * w2, the norm ahead of the output projection
// One workgroup per row; the row waits in LDS while the sums of squares of its
// runs are formed. Every run's sum is split over the same lanes whatever the
// batch is. A row at a negative position is inactive: zeros are written. All
// arithmetic is fp32.
#include "elem.h"

namespace kukeon {

DEV_INLINE void pn_ld4(const float* p, float* o) {
  const float4 a = *reinterpret_cast<const float4*>(p);
  o[0] = a.x; o[1] = a.y; o[2] = a.z; o[3] = a.w;
}
DEV_INLINE void pn_ld4(const bf16_t* p, float* o) {
  const uint2 a = *reinterpret_cast<const uint2*>(p);
  o[0] = us2f((unsigned short)(a.x & 0xffffu));
  o[1] = us2f((unsigned short)(a.x >> 16));
  o[2] = us2f((unsigned short)(a.y & 0xffffu));
  o[3] = us2f((unsigned short)(a.y >> 16));
}
DEV_INLINE void pn_st4(float* p, const float* v) {
  *reinterpret_cast<float4*>(p) = float4{v[0], v[1], v[2], v[3]};
}
DEV_INLINE void pn_st4(bf16_t* p, const float* v) {
  *reinterpret_cast<uint2*>(p) =
      uint2{(unsigned)f2us(v[0]) | ((unsigned)f2us(v[1]) << 16),
            (unsigned)f2us(v[2]) | ((unsigned)f2us(v[3]) << 16)};
}

// Partial sums of squares of the runs of su: red[g * SUB + k], SUB waves per
// run (or one wave after the other when there are more runs than waves).
DEV_INLINE void run_squares(const float* su, float* red, int groups, int part,
                            int SUB) {
  const int lane = threadIdx.x & (WAVE - 1);
  const int nw = blockDim.x / WAVE;
  for (int u = threadIdx.x / WAVE; u < groups * SUB; u += nw) {
    const int g = u / SUB, k = u - g * SUB;
    const float* s = su + (long)g * part;
    float ss = 0.f;
    for (int i = k * WAVE + lane; i < part; i += SUB * WAVE)
      ss = fmaf(s[i], s[i], ss);
    ss = wave_sum(ss);
    if (lane == 0) red[u] = ss;
  }
}
DEV_INLINE float run_scale(const float* red, int g, int SUB, int part,
                           float eps) {
  float s = 0.f;
  for (int k = 0; k < SUB; ++k) s += red[g * SUB + k];
  return 1.0f / sqrtf(s / (float)part + eps);
}

// V = 4: W and the run length are multiples of 4 and all rows 16-byte
// aligned (8 bytes for bf16), so a piece never straddles two runs.
template <typename T, int V, int NEXT>
__global__ __launch_bounds__(1024) void postnorm_kernel(
    float* __restrict__ x, const T* __restrict__ y, long ldy, float alpha,
    const float* __restrict__ scale, const float* __restrict__ w, int groups,
    float eps, int W, int SUB, const int* __restrict__ positions,
    T* __restrict__ h, const float* __restrict__ w2,
    const float* __restrict__ cw, int taps, float* __restrict__ state,
    const int* __restrict__ state_slots) {
  extern __shared__ float su[];          // [W], then groups * SUB sums
  float* red = su + W;
  const long r = blockIdx.x;
  const int p = positions[r];
  float* xr = x + r * (long)W;
  if (p < 0) {
    for (int i = threadIdx.x; i < W; i += blockDim.x) {
      xr[i] = 0.f;
      if (NEXT) stf(h + r * (long)W + i, 0.f);
    }
    return;
  }
  const T* yr = y + r * ldy;
  for (int i = threadIdx.x * V; i < W; i += blockDim.x * V) {
    float xv[V], yv[V], sv[V];
    if (V == 4) {
      pn_ld4(xr + i, xv); pn_ld4(yr + i, yv); pn_ld4(scale + i, sv);
    } else {
      xv[0] = xr[i]; yv[0] = ldf(yr + i); sv[0] = scale[i];
    }
#pragma unroll
    for (int k = 0; k < V; ++k) su[i + k] = fmaf(alpha, xv[k], sv[k] * yv[k]);
  }
  __syncthreads();
  const int part = W / groups;
  run_squares(su, red, groups, part, SUB);
  __syncthreads();
  const int back = taps - 1;
  float* st = NEXT == 1 ? state + (long)state_slots[r] * back * W : nullptr;
  for (int i = threadIdx.x * V; i < W; i += blockDim.x * V) {
    const float rs = run_scale(red, i / part, SUB, part, eps);
    float o[V], wv[V];
    if (V == 4) pn_ld4(w + i, wv);
    else wv[0] = w[i];
#pragma unroll
    for (int k = 0; k < V; ++k) o[k] = su[i + k] * rs * wv[k];
    if (V == 4) pn_st4(xr + i, o);
    else xr[i] = o[0];
    if (NEXT == 1) {
      // taps oldest first; entries before position 0 count as zero
      float acc[V];
#pragma unroll
      for (int k = 0; k < V; ++k) acc[k] = 0.f;
      for (int j = 0; j < taps; ++j) {
        if (p - back + j < 0) continue;
        float u[V], c[V];
        if (V == 4) {
          pn_ld4(cw + (long)j * W + i, c);
          if (j < back) pn_ld4(st + (long)j * W + i, u);
        } else {
          c[0] = cw[(long)j * W + i];
          if (j < back) u[0] = st[(long)j * W + i];
        }
#pragma unroll
        for (int k = 0; k < V; ++k)
          acc[k] = fmaf(c[k], j < back ? u[k] : o[k], acc[k]);
      }
      for (int j = 0; j < back; ++j) {
        if (V == 4) {
          float u[4];
          if (j + 1 < back) pn_ld4(st + (long)(j + 1) * W + i, u);
          pn_st4(st + (long)j * W + i, j + 1 < back ? u : o);
        } else {
          st[(long)j * W + i] = j + 1 < back ? st[(long)(j + 1) * W + i] : o[0];
        }
      }
      float hv[V];
#pragma unroll
      for (int k = 0; k < V; ++k) hv[k] = o[k] + acc[k];
      if (V == 4) pn_st4(h + r * (long)W + i, hv);
      else stf(h + r * (long)W + i, hv[0]);
    }
    if (NEXT == 2) {
      // the thread's own entries, read back by it below
#pragma unroll
      for (int k = 0; k < V; ++k) su[i + k] = o[k];
    }
  }
  if (NEXT == 2) {
    __syncthreads();
    run_squares(su, red, groups, part, SUB);
    __syncthreads();
    for (int i = threadIdx.x * V; i < W; i += blockDim.x * V) {
      const float rs = run_scale(red, i / part, SUB, part, eps);
      float o[V];
#pragma unroll
      for (int k = 0; k < V; ++k) o[k] = su[i + k] * rs * w2[i + k];
      if (V == 4) pn_st4(h + r * (long)W + i, o);
      else stf(h + r * (long)W + i, o[0]);
    }
  }
}

// x [T, W] fp32 in place; y [T, W] (stride(1) == 1); scale, w [W] fp32;
// positions [T]. next 0: h, w2, cw, state, state_slots are not read. next 1:
// h [T, W], cw [taps, W] fp32, state [slots, taps-1, W] fp32, state_slots [T]
// (row r is sequence r). next 2: h [T, W], w2 [W] fp32.
void postnorm_residual(torch::Tensor x, torch::Tensor y, double alpha,
                       torch::Tensor scale, torch::Tensor w, int64_t groups,
                       double eps, torch::Tensor positions, int64_t next,
                       torch::Tensor h, torch::Tensor w2, torch::Tensor cw,
                       torch::Tensor state, torch::Tensor state_slots) {
  check_f32(x, "x"); check_act(y, "y"); check_f32(scale, "scale");
  check_f32(w, "w"); check_i32(positions, "positions");
  TORCH_CHECK(x.dim() == 2 && y.dim() == 2 && y.stride(1) == 1);
  const long rows = x.size(0);
  const int W = (int)x.size(1);
  TORCH_CHECK(y.size(0) == rows && y.size(1) == W && scale.numel() == W &&
              w.numel() == W && positions.numel() == rows);
  TORCH_CHECK(groups >= 1 && W % groups == 0, "groups must divide the row");
  TORCH_CHECK(next >= 0 && next <= 2);
  long taps = 1;
  if (next) {
    TORCH_CHECK(h.is_cuda() && h.scalar_type() == y.scalar_type() &&
                h.dim() == 2 && h.is_contiguous() && h.size(0) == rows &&
                h.size(1) == W);
  }
  if (next == 1) {
    check_f32(cw, "cw"); check_f32(state, "state");
    check_i32(state_slots, "state_slots");
    taps = cw.size(0);
    TORCH_CHECK(cw.dim() == 2 && taps >= 1 && cw.size(1) == W);
    TORCH_CHECK(state.dim() == 3 && state.size(1) == taps - 1 &&
                state.size(2) == W && state_slots.numel() >= rows);
  }
  if (next == 2) {
    check_f32(w2, "w2");
    TORCH_CHECK(w2.numel() == W);
  }
  if (rows == 0) return;
  const int part = (int)(W / groups);
  bool vec = W % 4 == 0 && part % 4 == 0 && y.stride(0) % 4 == 0 &&
             aligned16(x.data_ptr()) && aligned16(y.data_ptr()) &&
             aligned16(scale.data_ptr()) && aligned16(w.data_ptr());
  if (next) vec = vec && aligned16(h.data_ptr());
  if (next == 1)
    vec = vec && aligned16(cw.data_ptr()) &&
          (taps == 1 || aligned16(state.data_ptr()));
  const int V = vec ? 4 : 1;
  int threads = (W / V + 63) / 64 * 64;
  threads = threads < 64 ? 64 : (threads > 1024 ? 1024 : threads);
  const int SUB = (int)std::max<long>(1, (threads / WAVE) / groups);
  const size_t shmem = ((size_t)W + (size_t)groups * SUB) * sizeof(float);
  TORCH_CHECK(shmem <= 64 * 1024, "row too wide for the LDS buffer");
  auto stream = c10::hip::getCurrentHIPStream().stream();
#define KK_GO(V_, N_)                                                          \
  {                                                                            \
    auto kern = postnorm_kernel<T, V_, N_>;                                    \
    static size_t allowed = 48 * 1024;                                         \
    if (shmem > allowed) {                                                     \
      hipFuncSetAttribute(reinterpret_cast<const void*>(kern),                 \
                          hipFuncAttributeMaxDynamicSharedMemorySize,          \
                          (int)shmem);                                         \
      allowed = shmem;                                                         \
    }                                                                          \
    kern<<<dim3((unsigned)rows), threads, shmem, stream>>>(                    \
        x.data_ptr<float>(), reinterpret_cast<const T*>(y.data_ptr()),         \
        (long)y.stride(0), (float)alpha, scale.data_ptr<float>(),              \
        w.data_ptr<float>(), (int)groups, (float)eps, W, SUB,                  \
        positions.data_ptr<int>(),                                             \
        next ? reinterpret_cast<T*>(h.data_ptr()) : nullptr,                   \
        next == 2 ? w2.data_ptr<float>() : nullptr,                            \
        next == 1 ? cw.data_ptr<float>() : nullptr, (int)taps,                 \
        next == 1 ? state.data_ptr<float>() : nullptr,                         \
        next == 1 ? state_slots.data_ptr<int>() : nullptr);                    \
  }
#define KK_NEXT(V_)                                                            \
  if (next == 0) KK_GO(V_, 0)                                                  \
  else if (next == 1) KK_GO(V_, 1)                                             \
  else KK_GO(V_, 2)
  KK_DISPATCH_ACT(y, {
    if (vec) { KK_NEXT(4) } else { KK_NEXT(1) }
  });
#undef KK_NEXT
#undef KK_GO
  HIP_CHECK_KERNEL();
}

}  // namespace kukeon
