// Python bindings for the delta kernel group: norms after the residual sum, in
// runs, fused with a causal convolution of the next input; the gated delta
// rule; the selective scan with a decay per channel and state; attention whose
// values are its unnormed keys, with per-head norms, a logarithmic distance
// bias and a sink; experts chosen by sigmoid scores. Built as its own module so
// that a model needing only these compiles nothing else.
#include <torch/extension.h>

namespace kukeon {
void embed_streams(torch::Tensor xs, torch::Tensor ids, torch::Tensor positions,
                   torch::Tensor table, torch::Tensor pos_table, double scale);
void postnorm_residual(torch::Tensor x, torch::Tensor y, double alpha,
                       torch::Tensor scale, torch::Tensor w, int64_t groups,
                       double eps, torch::Tensor positions, int64_t next,
                       torch::Tensor h, torch::Tensor w2, torch::Tensor cw,
                       torch::Tensor state, torch::Tensor state_slots);
void conv_act(torch::Tensor out, torch::Tensor proj, int64_t col0,
              torch::Tensor cw, torch::Tensor bias, torch::Tensor state,
              torch::Tensor positions, torch::Tensor row_seq,
              torch::Tensor cu_rows, torch::Tensor state_slots, int64_t act,
              bool shift_state, bool skip);
void conv_state_update(torch::Tensor state, torch::Tensor proj,
                       torch::Tensor bias, torch::Tensor positions,
                       torch::Tensor cu_rows, torch::Tensor state_slots,
                       int64_t q_col, int64_t k_col, int64_t v_col, int64_t Cq,
                       int64_t Ck, int64_t Cv);
void delta_scan(torch::Tensor y, torch::Tensor qkv, int64_t q_col,
                int64_t k_col, int64_t v_col, torch::Tensor ba, int64_t b_col,
                int64_t a_col, torch::Tensor rate, torch::Tensor dt_bias,
                double q_scale, torch::Tensor state, torch::Tensor positions,
                torch::Tensor cu_rows, torch::Tensor state_slots, int64_t H,
                int64_t G, int64_t d, int64_t dv);
void head_rmsnorm_gate(torch::Tensor out, torch::Tensor y, torch::Tensor gate,
                       torch::Tensor w, int64_t H, double eps, int64_t act,
                       double scale);
void selective_scan(torch::Tensor out, torch::Tensor x, torch::Tensor z,
                    torch::Tensor dt, torch::Tensor dt_bias, torch::Tensor bc,
                    int64_t b_col, int64_t c_col, torch::Tensor A2,
                    torch::Tensor D, torch::Tensor state,
                    torch::Tensor positions, torch::Tensor cu_rows,
                    torch::Tensor state_slots);
void head_norm_append(torch::Tensor q_out, torch::Tensor k_cache,
                      torch::Tensor proj, int64_t q_col, int64_t k_col,
                      torch::Tensor w, double eps, torch::Tensor positions,
                      torch::Tensor row_seq, torch::Tensor block_table);
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
void scaled_gate(torch::Tensor out, torch::Tensor a, torch::Tensor gate,
                 int64_t act, double scale);
void router_sigmoid(torch::Tensor idx, torch::Tensor wts, torch::Tensor logits,
                    int64_t top, double scale);
void routed_experts(torch::Tensor out, torch::Tensor h, torch::Tensor idx,
                    torch::Tensor wts, int64_t top, torch::Tensor w_gu,
                    torch::Tensor w_down, double limit, double alpha,
                    double shift, bool weigh_input, torch::Tensor extra);
void combine_rows_weighted(torch::Tensor out, torch::Tensor in,
                           torch::Tensor inv, torch::Tensor wts);
void clamp_glu(torch::Tensor out, torch::Tensor gate, torch::Tensor up,
               torch::Tensor bg, torch::Tensor bu, double limit, double alpha,
               double up_shift, torch::Tensor row_scale);
void gather_rows(torch::Tensor out, torch::Tensor in, torch::Tensor map);
bool chunk_attention_tiles_supported(int64_t d, int64_t dv, int64_t BS);
}  // namespace kukeon

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("embed_streams", &kukeon::embed_streams,
        "every stream = table[id] * scale + pos_table[position]");
  m.def("postnorm_residual", &kukeon::postnorm_residual,
        "x <- norm(alpha x + scale y) w, in runs, and what reads x next");
  m.def("conv_act", &kukeon::conv_act,
        "short causal convolution per channel, bias, activation, skip");
  m.def("conv_state_update", &kukeon::conv_state_update,
        "shift a portion's tail into the convolution state slots");
  m.def("delta_scan", &kukeon::delta_scan,
        "gated delta rule");
  m.def("head_rmsnorm_gate", &kukeon::head_rmsnorm_gate,
        "per head y / rms(y) * w * act(gate) * scale");
  m.def("selective_scan", &kukeon::selective_scan,
        "selective scan with a decay per channel and state, gated");
  m.def("head_norm_append", &kukeon::head_norm_append,
        "per-head query norm, paged append of the unnormed keys");
  m.def("masked_attention", &kukeon::masked_attention,
        "softmax attention with every mask, bias and sink");
  m.def("masked_attention_tiles", &kukeon::masked_attention_tiles,
        "the same for prompt portions on the matrix cores");
  m.def("scaled_gate", &kukeon::scaled_gate,
        "a * act(gate) * scale");
  m.def("router_sigmoid", &kukeon::router_sigmoid,
        "top experts by sigmoid scores, weights as they are");
  m.def("routed_experts", &kukeon::routed_experts,
        "the chosen experts of a small batch, by (row, choice) pairs");
  m.def("combine_rows_weighted", &kukeon::combine_rows_weighted,
        "out[t] = sum over k of w[t, k] * in[inv[t, k]]");
  m.def("clamp_glu", &kukeon::clamp_glu,
        "clamped gate * sigmoid(alpha gate) * (up + shift)");
  m.def("gather_rows", &kukeon::gather_rows,
        "out[r] = in[map[r]]");
  m.def("chunk_attention_tiles_supported",
        &kukeon::chunk_attention_tiles_supported);
}
