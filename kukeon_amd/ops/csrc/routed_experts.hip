// The chosen experts of a small batch, by (row, choice) pairs, with nothing
// leaving the device (a decode step can sit in a captured graph):
//   act[pair]  = glu(s W_gate[e] h_t, s W_up[e] h_t)      s: the pair's weight
//                where the weight multiplies the expert's INPUT, else 1
//   part[pair] = W_down[e] act[pair]                       fp32
//   out[t]     = sum_k w[t, k] part[t, k] (+ extra[t])     w = 1 where the
//                weight went in at the input; the k-th term added k-th
// glu is clamped gate * sigmoid(alpha gate) * (clamped up + shift) (no clamp,
// alpha 1 and shift 0: silu(gate) up).
//
// Two forms. Expert-major on the matrix cores (bf16, whole 16-byte pieces): a
// workgroup belongs to (expert, tile of output rows), lists the pairs routed to
// its expert and streams its weight rows past up to 32 of them at a time, so
// only the chosen experts leave HBM, once per step. Pair-major on the vector
// ALUs otherwise (any size, fp32): the input row waits in LDS, a wave owns
// output rows and its lanes stride over the reduction. A pair's sums are formed
// in an order fixed by the row length, never by the batch.
#include "elem.h"

namespace kukeon {

typedef __attribute__((__vector_size__(8 * sizeof(short)))) short re_bf16x8_v;
typedef __attribute__((__vector_size__(4 * sizeof(float)))) float re_f32x4_v;
DEV_INLINE re_bf16x8_v re_frag(const uint4& v) {
  return __builtin_bit_cast(re_bf16x8_v, v);
}

struct GluForm {
  float limit, alpha, shift;
};
DEV_INLINE float re_glu(float g, float u, const GluForm f) {
  g = fminf(g, f.limit);
  u = fminf(fmaxf(u, -f.limit), f.limit);
  return g / (1.0f + expf(-f.alpha * g)) * (u + f.shift);
}

#define RE_ROWS 8               // output rows per wave, pair-major form
#define RE_LIST 1024            // pairs of one expert listed at a time

// The pairs among [from, pairs) routed to expert e, in order, up to RE_LIST of
// them, by one wave into its own list; `from` moves to the first pair not
// looked at. -> how many.
DEV_INLINE int re_list(int* list, const int* __restrict__ idx, int ldi, int top,
                       int pairs, int e, int& from) {
  const int lane = threadIdx.x & (WAVE - 1);
  int n = 0;
  while (from < pairs && n + WAVE <= RE_LIST) {
    const int pair = from + lane;
    const bool mine = pair < pairs &&
                      idx[(long)(pair / top) * ldi + pair % top] == e;
    const unsigned long long m = __ballot(mine);
    if (mine) list[n + __popcll(m & ((1ull << lane) - 1ull))] = pair;
    n += __popcll(m);
    from += WAVE;
  }
  __builtin_amdgcn_wave_barrier();       // wave-private LDS, in order
  return n;
}

// A workgroup owns 16 gate rows and the 16 up rows beside them (UP), or 32 rows
// of W_down, of one expert. Its four waves share out the reduction in blocks of
// 128 entries (wave w takes blocks w, w + 4, ...), so a weight row is read once
// and an input row once per workgroup; v_mfma_f32_16x16x32_bf16 with the
// weights as A (lane = row, 8 consecutive k) and up to 32 listed pairs' rows as
// B; the waves' sums meet in LDS, added in wave order. Output lane (pair = l &
// 15) holds rows 4 (l >> 4) + r.
template <bool UP>
__global__ __launch_bounds__(256) void routed_mfma_kernel(
    void* __restrict__ dst, const bf16_t* __restrict__ src,
    const int* __restrict__ idx, int ldi, const float* __restrict__ wts, int ldw,
    const bf16_t* __restrict__ w, int NR, int wrows, int up_row, int K, int top,
    int pairs, int weigh, GluForm form) {
  __shared__ int lists[4][RE_LIST];
  __shared__ float sums[4][2][2][16 * 17];   // [wave][rows][pairs][pair, row]
  const int e = blockIdx.x;
  const int lane = threadIdx.x & (WAVE - 1);
  const int wave = threadIdx.x / WAVE;
  const int rc = lane & 15;
  const int g4 = lane >> 4;
  int* list = lists[wave];
  const int r0 = blockIdx.y * (UP ? 16 : 32);
  const int row0 = min(r0 + rc, NR - 1);
  const int row1 = UP ? up_row + row0 : min(r0 + 16 + rc, NR - 1);
  const bf16_t* wa = w + ((long)e * wrows + row0) * K + g4 * 8;
  const bf16_t* wb = w + ((long)e * wrows + row1) * K + g4 * 8;
  const uint4 zero = uint4{0u, 0u, 0u, 0u};
  int from = 0;
  while (from < pairs) {
    const int n = re_list(list, idx, ldi, top, pairs, e, from);
    for (int g0 = 0; g0 < n; g0 += 32) {
      const bool two = g0 + 16 < n;
      const int p0 = g0 + rc < n ? list[g0 + rc] : -1;
      const int p1 = g0 + 16 + rc < n ? list[g0 + 16 + rc] : -1;
      const bf16_t* x0 =
          src + (long)(p0 < 0 ? 0 : (UP ? p0 / top : p0)) * K + g4 * 8;
      const bf16_t* x1 =
          src + (long)(p1 < 0 ? 0 : (UP ? p1 / top : p1)) * K + g4 * 8;
      re_f32x4_v acc[2][2] = {{{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}},
                              {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}}};
#pragma unroll 2
      for (int k0 = wave * 128; k0 < K; k0 += 512) {
        uint4 a[4], b[4], x[4], z[4];
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int k = k0 + i * 32;
          const bool in = k + g4 * 8 < K;
          a[i] = in ? *reinterpret_cast<const uint4*>(wa + k) : zero;
          b[i] = in ? *reinterpret_cast<const uint4*>(wb + k) : zero;
          x[i] = in && p0 >= 0 ? *reinterpret_cast<const uint4*>(x0 + k) : zero;
          z[i] = zero;
        }
        if (two) {
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            const int k = k0 + i * 32;
            if (k + g4 * 8 < K && p1 >= 0)
              z[i] = *reinterpret_cast<const uint4*>(x1 + k);
          }
        }
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          acc[0][0] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              re_frag(a[i]), re_frag(x[i]), acc[0][0], 0, 0, 0);
          acc[1][0] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
              re_frag(b[i]), re_frag(x[i]), acc[1][0], 0, 0, 0);
        }
        if (two) {
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            acc[0][1] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                re_frag(a[i]), re_frag(z[i]), acc[0][1], 0, 0, 0);
            acc[1][1] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                re_frag(b[i]), re_frag(z[i]), acc[1][1], 0, 0, 0);
          }
        }
      }
      __syncthreads();                   // the previous sums are read
#pragma unroll
      for (int h = 0; h < 2; ++h)
#pragma unroll
        for (int q = 0; q < 2; ++q)
#pragma unroll
          for (int r = 0; r < 4; ++r)
            sums[wave][h][q][rc * 17 + 4 * g4 + r] = acc[h][q][r];
      __syncthreads();
      // thread -> (pair of the 32, row of the 16), two pairs per thread
#pragma unroll
      for (int q = 0; q < 2; ++q) {
        const int pi = threadIdx.x >> 4, row = threadIdx.x & 15;
        const int li = g0 + q * 16 + pi;
        if (li >= n) continue;
        const long pair = list[li];
        float s0 = 0.f, s1 = 0.f;
#pragma unroll
        for (int v = 0; v < 4; ++v) {
          s0 += sums[v][0][q][pi * 17 + row];
          s1 += sums[v][1][q][pi * 17 + row];
        }
        if (UP) {
          const float s =
              weigh ? wts[(pair / top) * ldw + pair % top] : 1.0f;
          if (r0 + row < NR)
            reinterpret_cast<bf16_t*>(dst)[pair * NR + r0 + row] =
                f2us(re_glu(s * s0, s * s1, form));
        } else {
          float* o = reinterpret_cast<float*>(dst) + pair * NR + r0 + row;
          if (r0 + row < NR) o[0] = s0;
          if (r0 + 16 + row < NR) o[16] = s1;
        }
      }
    }
  }
}

// Pair-major: blockIdx.x = pair, RE_ROWS output rows per wave.
template <typename T, bool UP>
__global__ __launch_bounds__(256) void routed_pair_kernel(
    void* __restrict__ dst, const T* __restrict__ src,
    const int* __restrict__ idx, int ldi, const float* __restrict__ wts, int ldw,
    const T* __restrict__ w, int NR, int wrows, int up_row, int K, int top,
    int weigh, GluForm form) {
  extern __shared__ float sx[];          // [K]
  const long pair = blockIdx.x;
  const long t = pair / top;
  const int kth = (int)(pair - t * top);
  const int e = idx[t * ldi + kth];
  const T* xr = src + (UP ? t : pair) * (long)K;
  for (int i = threadIdx.x; i < K; i += blockDim.x) sx[i] = ldf(xr + i);
  __syncthreads();
  const int lane = threadIdx.x & (WAVE - 1);
  const int f0 = (blockIdx.y * 4 + threadIdx.x / WAVE) * RE_ROWS;
  const float s = UP && weigh ? wts[t * ldw + kth] : 1.0f;
  for (int j = 0; j < RE_ROWS; ++j) {
    const int f = f0 + j;
    if (f >= NR) break;
    const T* wa = w + ((long)e * wrows + f) * K;
    const T* wb = wa + (long)up_row * K;
    float a = 0.f, b = 0.f;
    for (int i = lane; i < K; i += WAVE) {
      a = fmaf(ldf(wa + i), sx[i], a);
      if (UP) b = fmaf(ldf(wb + i), sx[i], b);
    }
    a = wave_sum(a);
    if (UP) b = wave_sum(b);
    if (lane == 0) {
      const long at = pair * NR + f;
      if (UP) stf(reinterpret_cast<T*>(dst) + at, re_glu(s * a, s * b, form));
      else reinterpret_cast<float*>(dst)[at] = a;
    }
  }
}

// out[t] = sum_k w[t, k] part[t * top + k] (+ extra[t])
template <typename T>
__global__ __launch_bounds__(256) void routed_fold_kernel(
    T* __restrict__ out, const float* __restrict__ part,
    const float* __restrict__ wts, int ldw, const T* __restrict__ extra,
    long total, int W, int top, int weigh) {
  const long i = (long)blockIdx.x * blockDim.x + threadIdx.x;
  if (i >= total) return;
  const long t = i / W;
  const int c = (int)(i - t * W);
  float acc = 0.f;
  for (int k = 0; k < top; ++k)
    acc = fmaf(weigh ? 1.0f : wts[t * ldw + k],
               part[(t * top + k) * (long)W + c], acc);
  if (extra) acc += ldf(extra + i);
  stf(out + i, acc);
}

// out, h [T, W]; idx [T, >= top] int32, wts [T, >= top] fp32 (row strides
// free); w_gu [E, 2 up_row, W]: gate rows from 0, up rows from up_row; w_down
// [E, W, ff]; extra [T, W] or empty. weigh_input: the weights multiply the
// experts' inputs and not their outputs.
void routed_experts(torch::Tensor out, torch::Tensor h, torch::Tensor idx,
                    torch::Tensor wts, int64_t top, torch::Tensor w_gu,
                    torch::Tensor w_down, double limit, double alpha,
                    double shift, bool weigh_input, torch::Tensor extra) {
  check_act(out, "out"); check_act(h, "h");
  TORCH_CHECK(h.dim() == 2 && h.is_contiguous() && out.is_contiguous() &&
              out.sizes() == h.sizes() && out.scalar_type() == h.scalar_type());
  const long rows = h.size(0);
  const int W = (int)h.size(1);
  TORCH_CHECK(idx.is_cuda() && idx.scalar_type() == torch::kInt32 &&
              wts.is_cuda() && wts.scalar_type() == torch::kFloat32 &&
              idx.dim() == 2 && wts.dim() == 2 && idx.stride(1) == 1 &&
              wts.stride(1) == 1 && idx.size(0) == rows && wts.size(0) == rows);
  TORCH_CHECK(top >= 1 && idx.size(1) >= top && wts.size(1) >= top);
  TORCH_CHECK(w_gu.dim() == 3 && w_down.dim() == 3 && w_gu.is_contiguous() &&
              w_down.is_contiguous() && w_gu.is_cuda() && w_down.is_cuda() &&
              w_gu.scalar_type() == h.scalar_type() &&
              w_down.scalar_type() == h.scalar_type());
  const long E = w_gu.size(0);
  const int wrows = (int)w_gu.size(1), up_row = wrows / 2;
  const int ff = (int)w_down.size(2);
  TORCH_CHECK(w_gu.size(2) == W && wrows % 2 == 0 && ff <= up_row &&
              w_down.size(0) == E && w_down.size(1) == W);
  const bool more = extra.numel() > 0;
  if (more)
    TORCH_CHECK(extra.is_cuda() && extra.is_contiguous() &&
                extra.sizes() == h.sizes() &&
                extra.scalar_type() == h.scalar_type());
  if (rows == 0) return;
  const long pairs = rows * top;
  TORCH_CHECK(pairs < (1L << 24));
  auto act = torch::empty({pairs, (long)ff}, h.options());
  auto part = torch::empty({pairs, (long)W},
                           h.options().dtype(torch::kFloat32));
  auto stream = c10::hip::getCurrentHIPStream().stream();
  const GluForm form{(float)limit, (float)alpha, (float)shift};
  const int ldi = (int)idx.stride(0), ldw = (int)wts.stride(0);
  const bool up_mfma = is_bf16(h) && W % 8 == 0 && aligned16(h.data_ptr()) &&
                       aligned16(w_gu.data_ptr());
  const bool down_mfma = is_bf16(h) && ff % 8 == 0 &&
                         aligned16(act.data_ptr()) &&
                         aligned16(w_down.data_ptr());
  TORCH_CHECK(up_mfma || (size_t)W * 4 <= 64 * 1024,
              "routed_experts: an input row does not fit LDS");
  TORCH_CHECK(down_mfma || (size_t)ff * 4 <= 64 * 1024,
              "routed_experts: an expert's row does not fit LDS");
  const int per = 4 * RE_ROWS;
  KK_DISPATCH_ACT(h, {
    if (up_mfma)
      routed_mfma_kernel<true><<<
          dim3((unsigned)E, (unsigned)((ff + 15) / 16)), 256, 0, stream>>>(
          act.data_ptr(), reinterpret_cast<const bf16_t*>(h.data_ptr()),
          idx.data_ptr<int>(), ldi, wts.data_ptr<float>(), ldw,
          reinterpret_cast<const bf16_t*>(w_gu.data_ptr()), ff, wrows, up_row,
          W, (int)top, (int)pairs, (int)weigh_input, form);
    else
      routed_pair_kernel<T, true><<<
          dim3((unsigned)pairs, (unsigned)((ff + per - 1) / per)), 256,
          (size_t)W * 4, stream>>>(
          act.data_ptr(), reinterpret_cast<const T*>(h.data_ptr()),
          idx.data_ptr<int>(), ldi, wts.data_ptr<float>(), ldw,
          reinterpret_cast<const T*>(w_gu.data_ptr()), ff, wrows, up_row, W,
          (int)top, (int)weigh_input, form);
    if (down_mfma)
      routed_mfma_kernel<false><<<
          dim3((unsigned)E, (unsigned)((W + 31) / 32)), 256, 0, stream>>>(
          part.data_ptr(), reinterpret_cast<const bf16_t*>(act.data_ptr()),
          idx.data_ptr<int>(), ldi, wts.data_ptr<float>(), ldw,
          reinterpret_cast<const bf16_t*>(w_down.data_ptr()), W, W, 0, ff,
          (int)top, (int)pairs, 0, form);
    else
      routed_pair_kernel<T, false><<<
          dim3((unsigned)pairs, (unsigned)((W + per - 1) / per)), 256,
          (size_t)ff * 4, stream>>>(
          part.data_ptr(), reinterpret_cast<const T*>(act.data_ptr()),
          idx.data_ptr<int>(), ldi, wts.data_ptr<float>(), ldw,
          reinterpret_cast<const T*>(w_down.data_ptr()), W, W, 0, ff, (int)top,
          0, form);
    const long total = rows * W;
    routed_fold_kernel<T><<<dim3((unsigned)((total + 255) / 256)), 256, 0,
                            stream>>>(
        reinterpret_cast<T*>(out.data_ptr()), part.data_ptr<float>(),
        wts.data_ptr<float>(), ldw,
        more ? reinterpret_cast<const T*>(extra.data_ptr()) : nullptr, total, W,
        (int)top, (int)weigh_input);
  });
  HIP_CHECK_KERNEL();
}

}  // namespace kukeon
