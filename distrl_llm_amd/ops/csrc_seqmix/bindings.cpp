// Python bindings of the sequence-mixing kernel library (gfx950).
#include <torch/extension.h>
#include <vector>

std::vector<torch::Tensor> offset_rmsnorm(torch::Tensor x, torch::Tensor w,
                                          double eps, bool out_bf16, double offset,
                                          int64_t groups);
void gated_residual_add(torch::Tensor x, torch::Tensor mix,
                        c10::optional<torch::Tensor> ff, torch::Tensor gates,
                        torch::Tensor gate_b, double mult);
std::vector<torch::Tensor> gated_residual_norm(
    torch::Tensor x, torch::Tensor mix, c10::optional<torch::Tensor> ff,
    torch::Tensor gates, torch::Tensor gate_b, double mult, torch::Tensor next_w,
    double eps, bool out_bf16);
torch::Tensor causal_tap_conv(torch::Tensor h, torch::Tensor w, torch::Tensor tails,
                              torch::Tensor cu, torch::Tensor tok_seq,
                              torch::Tensor slots, bool out_bf16);
torch::Tensor latent_prepare(torch::Tensor q, c10::optional<torch::Tensor> dkv, int64_t heads,
                             int64_t dim, int64_t rot_dim, int64_t kv_rank,
                             c10::optional<torch::Tensor> norm_w, double eps,
                             torch::Tensor positions, double rope_base,
                             int64_t rope_dims, torch::Tensor page_slot,
                             torch::Tensor cache, c10::optional<torch::Tensor> freqs,
                             double mag, bool pairs);
torch::Tensor latent_window_attention(torch::Tensor q_lat, torch::Tensor q_rot,
                                      torch::Tensor cache, int64_t kv_rank,
                                      torch::Tensor block_tables, int64_t block_size,
                                      torch::Tensor tok_seq, torch::Tensor positions,
                                      int64_t window, double scale,
                                      c10::optional<torch::Tensor> tiles,
                                      int64_t max_tile_queries,
                                      c10::optional<torch::Tensor> sink,
                                      c10::optional<torch::Tensor> gate);
torch::Tensor mingru_scan(torch::Tensor zxg, torch::Tensor bias, torch::Tensor state,
                          torch::Tensor cu, torch::Tensor slots,
                          c10::optional<torch::Tensor> chunks,
                          c10::optional<torch::Tensor> chunk_cu);
std::vector<torch::Tensor> moe_route(torch::Tensor h, torch::Tensor router_w,
                                     torch::Tensor router_b, int64_t top);
torch::Tensor moe_experts(torch::Tensor h, torch::Tensor idx, torch::Tensor wts,
                          torch::Tensor exp_gu, torch::Tensor exp_down);

std::vector<torch::Tensor> moe_route_all(torch::Tensor h, torch::Tensor router_w,
                                         c10::optional<torch::Tensor> correction,
                                         int64_t top, double scale, int64_t groups,
                                         int64_t keep_groups, bool renorm);
torch::Tensor moe_experts_relu2(torch::Tensor h, torch::Tensor idx, torch::Tensor wts,
                                torch::Tensor exp_up, torch::Tensor exp_down);
torch::Tensor moe_experts_glu(torch::Tensor h, torch::Tensor idx, torch::Tensor wts,
                              torch::Tensor exp_gu, torch::Tensor exp_down, double limit);
torch::Tensor tap_conv_silu(torch::Tensor x, torch::Tensor w, torch::Tensor tails,
                            torch::Tensor cu, torch::Tensor tok_seq, torch::Tensor slots,
                            bool out_bf16);
c10::optional<torch::Tensor> sandwich_residual_norm(
    torch::Tensor x, torch::Tensor y, c10::optional<torch::Tensor> y2,
    c10::optional<torch::Tensor> post_w, c10::optional<torch::Tensor> next_w, double eps,
    bool out_bf16, double offset, double y_scale, double y2_scale, bool cast_next,
    int64_t groups);
torch::Tensor gelu_tanh(torch::Tensor x);
std::vector<torch::Tensor> moe_route_sigmoid(torch::Tensor h, torch::Tensor router_w, int64_t top);
torch::Tensor moe_experts_scaled_input(torch::Tensor h, torch::Tensor idx, torch::Tensor wts,
                                       torch::Tensor exp_gu, torch::Tensor exp_down);
torch::Tensor qk_prepare_kv_write(torch::Tensor proj, int64_t heads, int64_t kv_heads, int64_t dim,
                                  int64_t vdim, c10::optional<torch::Tensor> q_norm_w,
                                  c10::optional<torch::Tensor> k_norm_w, double eps,
                                  torch::Tensor positions, c10::optional<torch::Tensor> freqs,
                                  double mag, c10::optional<torch::Tensor> mix,
                                  torch::Tensor page_slot, torch::Tensor cache, int64_t maps,
                                  bool unit, double temp_coef, double temp_every,
                                  c10::optional<torch::Tensor> conv_w,
                                  c10::optional<torch::Tensor> tails,
                                  c10::optional<torch::Tensor> cu,
                                  c10::optional<torch::Tensor> tok_seq,
                                  c10::optional<torch::Tensor> slots);
torch::Tensor window_attention(torch::Tensor q, torch::Tensor cache, int64_t heads,
                               int64_t kv_heads, int64_t dim, int64_t vdim, bool whole_key,
                               torch::Tensor block_tables, int64_t block_size,
                               torch::Tensor tok_seq, torch::Tensor positions, double scale,
                               int64_t window, int64_t keep_first,
                               c10::optional<torch::Tensor> r1, c10::optional<torch::Tensor> r2,
                               c10::optional<torch::Tensor> gate,
                               c10::optional<torch::Tensor> tiles, int64_t max_tile_queries,
                               int64_t maps, c10::optional<torch::Tensor> lam_w, double diff,
                               double eps, int64_t chunk, double softcap,
                               c10::optional<torch::Tensor> sink);
std::vector<torch::Tensor> parallel_start(torch::Tensor embed, torch::Tensor tokens, double scale,
                                          c10::optional<torch::Tensor> step, torch::Tensor norm_w,
                                          double eps, bool out_bf16, double offset);
c10::optional<torch::Tensor> parallel_residual_norm(
    torch::Tensor x, c10::optional<torch::Tensor> y, c10::optional<torch::Tensor> y2,
    c10::optional<torch::Tensor> y_w, c10::optional<torch::Tensor> y2_w, double y_scale,
    double y2_scale, c10::optional<torch::Tensor> f, c10::optional<torch::Tensor> embed,
    c10::optional<torch::Tensor> tokens, double scale, c10::optional<torch::Tensor> step,
    c10::optional<torch::Tensor> norm_w, double eps, bool out_bf16, double offset);
torch::Tensor linear_attention(torch::Tensor proj, int64_t heads, int64_t dim, int64_t vdim,
                               torch::Tensor powers, torch::Tensor norm_w, double eps,
                               torch::Tensor state, torch::Tensor cu, torch::Tensor slots,
                               int64_t max_tile);
torch::Tensor linear_unit(torch::Tensor proj, torch::Tensor conv_w, torch::Tensor conv_b,
                          torch::Tensor tails, torch::Tensor gates_w, torch::Tensor gates_b,
                          torch::Tensor lam, double c, torch::Tensor state, torch::Tensor cu,
                          torch::Tensor tok_seq, torch::Tensor slots,
                          c10::optional<torch::Tensor> tiles, c10::optional<torch::Tensor> tile_cu);
torch::Tensor gelu_glu(torch::Tensor gu);
torch::Tensor cap_logits(torch::Tensor z, double scale, double cap);
std::vector<torch::Tensor> hyper_start(torch::Tensor embed, torch::Tensor tokens, double scale,
                                       int64_t streams, torch::Tensor read_w, torch::Tensor norm_w,
                                       double eps, bool out_bf16, bool center);
c10::optional<torch::Tensor> hyper_residual_norm(
    torch::Tensor x, torch::Tensor y, c10::optional<torch::Tensor> y2,
    c10::optional<torch::Tensor> y_w, c10::optional<torch::Tensor> y2_w, double y_scale,
    double y2_scale, torch::Tensor mix, torch::Tensor out_w, c10::optional<torch::Tensor> read_w,
    c10::optional<torch::Tensor> norm_w, double eps, bool out_bf16, bool center);
torch::Tensor hyper_close_norm(torch::Tensor x, torch::Tensor rows, torch::Tensor norm_w, double eps,
                               bool out_bf16, bool center);
torch::Tensor capped_glu(torch::Tensor gu, double limit);
torch::Tensor silu_glu(torch::Tensor gu);
torch::Tensor qk_norm_kv_write(torch::Tensor proj, int64_t heads, int64_t kv_heads, int64_t dim,
                               int64_t vdim, torch::Tensor q_norm_w, torch::Tensor k_norm_w,
                               double eps, torch::Tensor page_slot, torch::Tensor cache);
torch::Tensor sigmoid_attention(torch::Tensor q, torch::Tensor cache, int64_t heads,
                                int64_t kv_heads, int64_t dim, int64_t vdim,
                                torch::Tensor block_tables, int64_t block_size,
                                torch::Tensor tok_seq, torch::Tensor positions, double scale,
                                int64_t window, int64_t keep_first, torch::Tensor slopes,
                                torch::Tensor pos_bias, c10::optional<torch::Tensor> tiles,
                                int64_t max_tile_queries);
torch::Tensor rope_kv_write(torch::Tensor proj, int64_t heads, int64_t kv_heads, int64_t dim,
                            int64_t vdim, torch::Tensor positions, double rope_base,
                            int64_t rope_dims, torch::Tensor page_slot, torch::Tensor cache,
                            c10::optional<torch::Tensor> vmix,
                            c10::optional<torch::Tensor> v_first);
torch::Tensor sink_attention(torch::Tensor q, torch::Tensor cache, int64_t heads,
                             int64_t kv_heads, int64_t dim, int64_t vdim,
                             torch::Tensor block_tables, int64_t block_size,
                             torch::Tensor tok_seq, torch::Tensor positions, double scale,
                             double softcap, c10::optional<torch::Tensor> sink,
                             c10::optional<torch::Tensor> talk,
                             c10::optional<torch::Tensor> tiles, int64_t max_tile_queries);
torch::Tensor gated_delta_rule(torch::Tensor qkv, torch::Tensor gate,
                               c10::optional<torch::Tensor> ab,
                               c10::optional<torch::Tensor> h,
                               c10::optional<torch::Tensor> ab_w, torch::Tensor a_log, torch::Tensor dt_bias, torch::Tensor onorm_w,
                               double eps, torch::Tensor state, torch::Tensor cu,
                               torch::Tensor slots, int64_t heads, int64_t kv_heads,
                               int64_t dim, int64_t vdim,
                               c10::optional<torch::Tensor> decay_up, bool gate_sigmoid);

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("offset_rmsnorm", &offset_rmsnorm, "offset-weight RMS norm -> (fp32, dtype)");
  m.def("gated_residual_add", &gated_residual_add, "gated parallel-residual update");
  m.def("gated_residual_norm", &gated_residual_norm,
        "gated residual update fused with the next offset RMS norm");
  m.def("causal_tap_conv", &causal_tap_conv, "short causal depthwise conv with slot tails");
  m.def("latent_prepare", &latent_prepare, "latent cache write + query rotation");
  m.def("latent_window_attention", &latent_window_attention,
        "windowed paged attention in latent space");
  m.def("mingru_scan", &mingru_scan, "minGRU scan with per-slot fp32 state");
  m.def("moe_route", &moe_route, "fp32 top-k router");
  m.def("moe_experts", &moe_experts, "grouped-GEMM mixture of SiLU-gated experts");
  m.def("moe_route_all", &moe_route_all, "fp32 router: softmax over all, corrected choice");
  m.def("moe_experts_glu", &moe_experts_glu,
        "grouped-GEMM mixture of clamped-GLU experts with identity experts");
  m.def("tap_conv_silu", &tap_conv_silu, "short causal conv + SiLU with slot tails");
  m.def("sandwich_residual_norm", &sandwich_residual_norm,
        "closing norm + residual sum + next opening norm");
  m.def("capped_glu", &capped_glu, "clamped GLU activation");
  m.def("silu_glu", &silu_glu, "SiLU-gated GLU activation");
  m.def("qk_norm_kv_write", &qk_norm_kv_write, "per-head RMS norm of q/k, K/V cache write");
  m.def("sigmoid_attention", &sigmoid_attention,
        "paged GQA with sigmoid weights, distance penalty, window with kept first tokens");
  m.def("rope_kv_write", &rope_kv_write, "pair rotary on q/k, value blend, K/V cache write");
  m.def("sink_attention", &sink_attention,
        "paged GQA with capped scores, sinks and head mixing");
  m.def("gated_delta_rule", &gated_delta_rule, "gated delta rule with per-slot fp32 state");
  m.def("gelu_tanh", &gelu_tanh, "tanh-form GELU activation");
  m.def("moe_route_sigmoid", &moe_route_sigmoid, "fp32 router: sigmoid scores, top-k, no renormalisation");
  m.def("moe_experts_scaled_input", &moe_experts_scaled_input,
        "grouped-GEMM mixture of SiLU-gated experts whose input carries the routing weight");
  m.def("qk_prepare_kv_write", &qk_prepare_kv_write,
        "short conv, q/k norm, half rotary, query temperature, score-mixing fold, K/V cache write");
  m.def("gelu_glu", &gelu_glu, "tanh-GELU-gated GLU activation");
  m.def("cap_logits", &cap_logits, "scaled, tanh-capped fp32 logits");
  m.def("hyper_start", &hyper_start, "embedding into residual streams + first norm");
  m.def("hyper_residual_norm", &hyper_residual_norm,
        "stream update of a sublayer's output + next read sum and norm");
  m.def("hyper_close_norm", &hyper_close_norm, "norm of the streams' sum");
  m.def("moe_experts_relu2", &moe_experts_relu2, "grouped-GEMM mixture of squared-ReLU experts");
  m.def("parallel_start", &parallel_start, "scaled embedding rows + first norm");
  m.def("parallel_residual_norm", &parallel_residual_norm,
        "parallel block's layer tail: normed sides, feed-forward, pass injection, next norm");
  m.def("linear_attention", &linear_attention,
        "linear attention with fixed decays, fp32 state per slot, gated RMS norm");
  m.def("linear_unit", &linear_unit, "real-gated linear recurrent unit with short convolution");
  m.def("window_attention", &window_attention,
        "paged GQA softmax attention: window or chunks, kept first tokens, log distance bias, cap, sink, two maps, output gate");
}
