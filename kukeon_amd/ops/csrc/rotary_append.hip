// Query/key preparation of grouped-query attention with partial rotary
// positions over a packed batch:
//   q_out[r, h, :]  = rotated query of head h
//   key page row    = rotated key, value page row = value as projected
// The first `dims` entries of every query and key head turn as pairs
// (2i, 2i+1) by the angle table row cs[position] = [cos_0 .. | sin_0 ..]; the
// others pass. Angles, products and sums are fp32.
#include "elem.h"

namespace kukeon {

// blockIdx.x = row, the row's pieces over blockIdx.y and the threads. VEC: a
// piece is 8 entries of one head (16-byte accesses); otherwise one entry, read
// together with its partner.
template <typename T, bool VEC>
__global__ __launch_bounds__(256) void rotary_append_kernel(
    T* __restrict__ q_out, T* __restrict__ k_cache, T* __restrict__ v_cache,
    const T* __restrict__ proj, long ldp, long q_col, long k_col, long v_col,
    const float* __restrict__ cs, int cs_rows, int dims,
    const int* __restrict__ positions, const int* __restrict__ row_seq,
    const int* __restrict__ block_table, int max_blocks, int H, int G, int d,
    int dv, int BS) {
  constexpr int N = VEC ? 8 : 1;
  const int Cq = H * d, Ck = G * d, Cv = G * dv;
  const long r = blockIdx.x;
  const int p = positions[r];
  int c = (int)(blockIdx.y * blockDim.x + threadIdx.x) * N;
  if (p < 0 || c >= Cq + Ck + Cv) return;
  const T* row = proj + r * ldp;
  const T* src;
  T* dst;
  int e;                       // entry within its head
  bool turn = true;
  if (c < Cq) {
    src = row + q_col + c;
    dst = q_out + r * (long)Cq + c;
    e = c % d;
  } else {
    const long blk = block_table[(long)row_seq[r] * max_blocks + p / BS];
    const int at = p % BS;
    c -= Cq;
    if (c < Ck) {
      const int g = c / d;
      e = c - g * d;
      src = row + k_col + c;
      dst = k_cache + ((blk * G + g) * BS + at) * (long)d + e;
    } else {
      c -= Ck;
      const int g = c / dv;
      e = c - g * dv;
      src = row + v_col + c;
      dst = v_cache + ((blk * G + g) * BS + at) * (long)dv + e;
      turn = false;
    }
  }
  const float* ang = cs + (long)(p < cs_rows ? p : cs_rows - 1) * dims;
  const int half = dims / 2;
  if (VEC) {
    if (!turn || e >= dims) {
      Raw8<T> v;
      v.load(src);
      *reinterpret_cast<Raw8<T>*>(dst) = v;
      return;
    }
    float v[8];
    ld8(src, v);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int e0 = e + 2 * i;
      if (e0 < dims) {
        const float co = ang[e0 >> 1], sn = ang[half + (e0 >> 1)];
        const float a = v[2 * i], b = v[2 * i + 1];
        v[2 * i] = fmaf(a, co, -b * sn);
        v[2 * i + 1] = fmaf(b, co, a * sn);
      }
    }
    st8(dst, v);
  } else {
    float v = ldf(src);
    if (turn && e < dims) {
      const float other = ldf((e & 1) ? src - 1 : src + 1);
      const float co = ang[e >> 1], sn = ang[half + (e >> 1)];
      v = (e & 1) ? fmaf(v, co, other * sn) : fmaf(v, co, -other * sn);
    }
    stf(dst, v);
  }
}

// q_out [T, H*d] contiguous; k_cache [blocks, G, BS, d], v_cache [blocks, G,
// BS, dv]; proj [T, ld] (stride(1) == 1) with the three segments at their
// columns; cs [positions, dims] fp32.
void rotary_append(torch::Tensor q_out, torch::Tensor k_cache,
                   torch::Tensor v_cache, torch::Tensor proj, int64_t q_col,
                   int64_t k_col, int64_t v_col, torch::Tensor cs,
                   torch::Tensor positions, torch::Tensor row_seq,
                   torch::Tensor block_table) {
  check_act(proj, "proj");
  check_i32(positions, "positions"); check_i32(row_seq, "row_seq");
  check_i32(block_table, "block_table");
  TORCH_CHECK(proj.dim() == 2 && proj.stride(1) == 1);
  TORCH_CHECK(cs.is_cuda() && cs.scalar_type() == torch::kFloat32 &&
              cs.dim() == 2 && cs.is_contiguous() && cs.size(0) >= 1 &&
              cs.size(1) % 2 == 0);
  const long rows = proj.size(0);
  TORCH_CHECK(k_cache.dim() == 4 && k_cache.is_contiguous() &&
              v_cache.dim() == 4 && v_cache.is_contiguous() &&
              k_cache.scalar_type() == proj.scalar_type() &&
              v_cache.scalar_type() == proj.scalar_type());
  const int G = (int)k_cache.size(1), BS = (int)k_cache.size(2);
  const int d = (int)k_cache.size(3), dv = (int)v_cache.size(3);
  const int dims = (int)cs.size(1);
  TORCH_CHECK(v_cache.size(0) == k_cache.size(0) && v_cache.size(1) == G &&
              v_cache.size(2) == BS && dims <= d);
  TORCH_CHECK(q_out.dim() == 2 && q_out.is_contiguous() &&
              q_out.size(0) == rows && q_out.size(1) % d == 0 &&
              q_out.scalar_type() == proj.scalar_type());
  const int H = (int)(q_out.size(1) / d);
  TORCH_CHECK(q_col >= 0 && q_col + (long)H * d <= proj.size(1) &&
              k_col >= 0 && k_col + (long)G * d <= proj.size(1) &&
              v_col >= 0 && v_col + (long)G * dv <= proj.size(1));
  TORCH_CHECK(positions.numel() == rows && row_seq.numel() == rows);
  TORCH_CHECK(block_table.dim() == 2);
  if (rows == 0) return;
  const bool vec = d % 8 == 0 && dv % 8 == 0 && q_col % 8 == 0 &&
                   k_col % 8 == 0 && v_col % 8 == 0 &&
                   proj.stride(0) % 8 == 0 && aligned16(proj.data_ptr()) &&
                   aligned16(q_out.data_ptr()) &&
                   aligned16(k_cache.data_ptr()) &&
                   aligned16(v_cache.data_ptr());
  const long per = ((long)H * d + (long)G * (d + dv)) / (vec ? 8 : 1);
  TORCH_CHECK(per <= 65535L * 256);
  auto stream = c10::hip::getCurrentHIPStream().stream();
  dim3 grid((unsigned)rows, (unsigned)((per + 255) / 256));
#define KK_ARGS reinterpret_cast<T*>(q_out.data_ptr()),                        \
        reinterpret_cast<T*>(k_cache.data_ptr()),                              \
        reinterpret_cast<T*>(v_cache.data_ptr()),                              \
        reinterpret_cast<const T*>(proj.data_ptr()), (long)proj.stride(0),     \
        (long)q_col, (long)k_col, (long)v_col, cs.data_ptr<float>(),           \
        (int)cs.size(0), dims, positions.data_ptr<int>(),                      \
        row_seq.data_ptr<int>(), block_table.data_ptr<int>(),                  \
        (int)block_table.size(1), H, G, d, dv, BS
  KK_DISPATCH_ACT(proj, {
    if (vec) rotary_append_kernel<T, true><<<grid, 256, 0, stream>>>(KK_ARGS);
    else rotary_append_kernel<T, false><<<grid, 256, 0, stream>>>(KK_ARGS);
  });
#undef KK_ARGS
  HIP_CHECK_KERNEL();
}

}  // namespace kukeon
