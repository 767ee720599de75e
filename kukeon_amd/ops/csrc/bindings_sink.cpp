// Python bindings for the sink kernel group: embedding rows normed on their way
// into an fp32 residual stream, partial rotary positions with the page write,
// attention over a window and kept first tokens and latent attention, both with
// a sink per head in the softmax, experts chosen by corrected sigmoid scores in
// groups. Built as its own module so that a model needing only these compiles
// nothing else.
#include <torch/extension.h>

namespace kukeon {
void embed_rmsnorm(torch::Tensor x, torch::Tensor out, torch::Tensor ids,
                   torch::Tensor table, torch::Tensor w, torch::Tensor w2,
                   double w_offset, double eps);
void residual_add_rmsnorm(torch::Tensor x, torch::Tensor a, torch::Tensor bias,
                          torch::Tensor w, double w_offset, double eps,
                          torch::Tensor out);
void rotary_append(torch::Tensor q_out, torch::Tensor k_cache,
                   torch::Tensor v_cache, torch::Tensor proj, int64_t q_col,
                   int64_t k_col, int64_t v_col, torch::Tensor cs,
                   torch::Tensor positions, torch::Tensor row_seq,
                   torch::Tensor block_table);
void masked_attention(torch::Tensor out, torch::Tensor q, torch::Tensor k_cache,
                      torch::Tensor v_cache, torch::Tensor slopes,
                      torch::Tensor r1, torch::Tensor r2, torch::Tensor sinks,
                      torch::Tensor positions, torch::Tensor row_seq,
                      torch::Tensor block_table, int64_t H, double scale,
                      double softcap, int64_t chunk, int64_t window,
                      int64_t keep, double key_eps);
void masked_attention_tiles(torch::Tensor out, torch::Tensor q,
                            torch::Tensor k_cache, torch::Tensor v_cache,
                            torch::Tensor r1, torch::Tensor r2,
                            torch::Tensor sinks, torch::Tensor block_table,
                            torch::Tensor seq_lens, torch::Tensor q_starts,
                            torch::Tensor qb_seq, torch::Tensor qb_start,
                            double scale, double softcap, int64_t chunk,
                            int64_t window, int64_t keep, double key_eps);
bool chunk_attention_tiles_supported(int64_t d, int64_t dv, int64_t BS);
void latent_kv_append(torch::Tensor cq_out, torch::Tensor cache,
                      torch::Tensor proj, int64_t q_col, int64_t kv_col,
                      torch::Tensor wq, torch::Tensor wkv, double eps,
                      torch::Tensor cs, torch::Tensor positions,
                      torch::Tensor row_seq, torch::Tensor block_table);
void latent_attention(torch::Tensor out, torch::Tensor q_abs, torch::Tensor q,
                      torch::Tensor cache, torch::Tensor cs,
                      torch::Tensor positions, torch::Tensor row_seq,
                      torch::Tensor block_table, int64_t H, int64_t dn,
                      int64_t dr, int64_t window, double scale,
                      torch::Tensor sinks);
void head_gate(torch::Tensor out, torch::Tensor o, torch::Tensor gate);
void router_corrected(torch::Tensor idx, torch::Tensor wts,
                      torch::Tensor logits, torch::Tensor correction,
                      int64_t top, int64_t groups, int64_t keep, int64_t best,
                      double scale, bool renorm);
void routed_experts(torch::Tensor out, torch::Tensor h, torch::Tensor idx,
                    torch::Tensor wts, int64_t top, torch::Tensor w_gu,
                    torch::Tensor w_down, double limit, double alpha,
                    double shift, bool weigh_input, torch::Tensor extra);
void clamp_glu(torch::Tensor out, torch::Tensor gate, torch::Tensor up,
               torch::Tensor bg, torch::Tensor bu, double limit, double alpha,
               double up_shift, torch::Tensor row_scale);
void combine_rows_weighted(torch::Tensor out, torch::Tensor in,
                           torch::Tensor inv, torch::Tensor wts);
void gather_rows(torch::Tensor out, torch::Tensor in, torch::Tensor map);
void relu_square_(torch::Tensor x);
}  // namespace kukeon

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("embed_rmsnorm", &kukeon::embed_rmsnorm,
        "x = rmsnorm(table[id]) * w, out = rmsnorm(x) * w2");
  m.def("residual_add_rmsnorm", &kukeon::residual_add_rmsnorm,
        "x += a; out = rmsnorm(x) * (w_offset + w)");
  m.def("rotary_append", &kukeon::rotary_append,
        "rotate queries and keys in part, paged K/V append");
  m.def("masked_attention", &kukeon::masked_attention,
        "softmax attention over paged keys with every option of the row kernel");
  m.def("masked_attention_tiles", &kukeon::masked_attention_tiles,
        "the same for prompt portions on the matrix cores");
  m.def("chunk_attention_tiles_supported",
        &kukeon::chunk_attention_tiles_supported);
  m.def("latent_kv_append", &kukeon::latent_kv_append,
        "norm the latents, rotate the shared key part, write the cache row");
  m.def("latent_attention", &kukeon::latent_attention,
        "attention over the shared latent cache row");
  m.def("head_gate", &kukeon::head_gate,
        "[H,T,dv] -> [T,H*dv], with or without a sigmoid gate");
  m.def("router_corrected", &kukeon::router_corrected,
        "sigmoid scores, choice by corrected scores within the best groups");
  m.def("routed_experts", &kukeon::routed_experts,
        "the chosen experts of a small batch, by (row, choice) pairs");
  m.def("clamp_glu", &kukeon::clamp_glu,
        "clamped gate * sigmoid(alpha gate) * (up + shift)");
  m.def("combine_rows_weighted", &kukeon::combine_rows_weighted,
        "out[t] = sum over k of w[t, k] * in[inv[t, k]]");
  m.def("gather_rows", &kukeon::gather_rows, "out[r] = in[map[r]]");
  m.def("relu_square_", &kukeon::relu_square_, "x = max(x, 0)^2 in place");
}
