// Query/key preparation of an attention that norms each head by itself and
// keeps ONE unnormed key row per token and kv head, its values being the keys
// as projected:
//   q[r, h, :]  = q / rms(q) * w          per head, w [d] shared by the heads
//   page row    = k                       as projected
// The score needs the normed key k / rms(k) * w_k; the attention kernels take
// rms(k) from the row they read anyway, and w_k can wait on the query side,
// (q w_q) . (k / rms(k) w_k) = (q w_q w_k) . k / rms(k), so w is the product
// of both weights and the page row serves as key and as value.
#include "elem.h"

namespace kukeon {

// One unit per (row, head); heads H .. H + G - 1 are the key heads. VEC: LP
// lanes (a power of two) per unit, 8 entries each, lanes past d / 8 idle.
// Otherwise a wave per unit whose lanes stride over the entries.
template <typename T, bool VEC>
__global__ __launch_bounds__(256) void head_norm_append_kernel(
    T* __restrict__ q_out, T* __restrict__ k_cache, const T* __restrict__ proj,
    long ldp, long q_col, long k_col, const float* __restrict__ w, float eps,
    const int* __restrict__ positions, const int* __restrict__ row_seq,
    const int* __restrict__ block_table, int max_blocks, long rows, int H,
    int G, int d, int BS, int LP) {
  const long t = (long)blockIdx.x * blockDim.x + threadIdx.x;
  const long unit = t / LP;
  const int sub = (int)(t - unit * LP);
  const int NH = H + G;
  const bool inside = unit < rows * NH;
  const long r = inside ? unit / NH : 0;
  const int hd = inside ? (int)(unit - r * NH) : 0;
  const int p = positions[r];
  const bool live = inside && p >= 0;
  const bool isq = hd < H;
  const T* src = proj + r * ldp +
                 (isq ? q_col + (long)hd * d : k_col + (long)(hd - H) * d);
  T* dst;
  if (isq || !live) {
    dst = q_out + (r * H + (isq ? hd : 0)) * (long)d;
  } else {
    const long blk = block_table[(long)row_seq[r] * max_blocks + p / BS];
    dst = k_cache + ((blk * G + (hd - H)) * BS + p % BS) * (long)d;
  }
  if (VEC) {
    const bool has = live && sub * 8 < d;
    float v[8];
#pragma unroll
    for (int k = 0; k < 8; ++k) v[k] = 0.f;
    if (has) ld8(src + sub * 8, v);
    float ss = 0.f;
#pragma unroll
    for (int k = 0; k < 8; ++k) ss = fmaf(v[k], v[k], ss);
    for (int off = LP >> 1; off > 0; off >>= 1) ss += __shfl_xor(ss, off, WAVE);
    if (!has) return;
    if (isq) {
      const float rs = 1.0f / sqrtf(ss / (float)d + eps);
      float ww[8];
      ld8(w + sub * 8, ww);
#pragma unroll
      for (int k = 0; k < 8; ++k) v[k] = v[k] * rs * ww[k];
    }
    st8(dst + sub * 8, v);
  } else {
    float ss = 0.f;
    if (live)
      for (int i = sub; i < d; i += LP) {
        const float v = ldf(src + i);
        ss = fmaf(v, v, ss);
      }
    ss = wave_sum(ss);
    if (!live) return;
    const float rs = 1.0f / sqrtf(ss / (float)d + eps);
    for (int i = sub; i < d; i += LP) {
      const float v = ldf(src + i);
      stf(dst + i, isq ? v * rs * w[i] : v);
    }
  }
}

// q_out [T, H*d] contiguous; k_cache [blocks, G, BS, d]; proj [T, ld]
// (stride(1) == 1); w [d] fp32.
void head_norm_append(torch::Tensor q_out, torch::Tensor k_cache,
                      torch::Tensor proj, int64_t q_col, int64_t k_col,
                      torch::Tensor w, double eps, torch::Tensor positions,
                      torch::Tensor row_seq, torch::Tensor block_table) {
  check_act(proj, "proj"); check_f32(w, "w");
  check_i32(positions, "positions"); check_i32(row_seq, "row_seq");
  check_i32(block_table, "block_table");
  TORCH_CHECK(proj.dim() == 2 && proj.stride(1) == 1);
  const long rows = proj.size(0);
  TORCH_CHECK(k_cache.dim() == 4 && k_cache.is_contiguous() &&
              k_cache.scalar_type() == proj.scalar_type());
  const int G = (int)k_cache.size(1), BS = (int)k_cache.size(2);
  const int d = (int)k_cache.size(3);
  TORCH_CHECK(w.numel() == d);
  TORCH_CHECK(q_out.dim() == 2 && q_out.is_contiguous() &&
              q_out.size(0) == rows && q_out.size(1) % d == 0 &&
              q_out.scalar_type() == proj.scalar_type());
  const int H = (int)(q_out.size(1) / d);
  TORCH_CHECK(q_col >= 0 && q_col + (long)H * d <= proj.size(1) &&
              k_col >= 0 && k_col + (long)G * d <= proj.size(1));
  TORCH_CHECK(positions.numel() == rows && row_seq.numel() == rows);
  TORCH_CHECK(block_table.dim() == 2);
  if (rows == 0) return;
  const bool vec = d % 8 == 0 && d <= 8 * WAVE && q_col % 8 == 0 &&
                   k_col % 8 == 0 && proj.stride(0) % 8 == 0 &&
                   aligned16(proj.data_ptr()) && aligned16(q_out.data_ptr()) &&
                   aligned16(k_cache.data_ptr()) && aligned16(w.data_ptr());
  int LP = WAVE;
  if (vec) {
    LP = 1;
    while (LP * 8 < d) LP <<= 1;
  }
  const long threads = rows * (H + G) * LP;
  auto stream = c10::hip::getCurrentHIPStream().stream();
  dim3 grid((unsigned)((threads + 255) / 256));
#define KK_ARGS reinterpret_cast<T*>(q_out.data_ptr()),                        \
        reinterpret_cast<T*>(k_cache.data_ptr()),                              \
        reinterpret_cast<const T*>(proj.data_ptr()), (long)proj.stride(0),     \
        (long)q_col, (long)k_col, w.data_ptr<float>(), (float)eps,             \
        positions.data_ptr<int>(), row_seq.data_ptr<int>(),                    \
        block_table.data_ptr<int>(), (int)block_table.size(1), rows, H, G, d,  \
        BS, LP
  KK_DISPATCH_ACT(proj, {
    if (vec) head_norm_append_kernel<T, true><<<grid, 256, 0, stream>>>(KK_ARGS);
    else head_norm_append_kernel<T, false><<<grid, 256, 0, stream>>>(KK_ARGS);
  });
#undef KK_ARGS
  HIP_CHECK_KERNEL();
}

}  // namespace kukeon
