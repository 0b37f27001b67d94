// pybind11 bindings for the token-batch kernel library (_hip_lm.so).
#include <torch/extension.h>

using Opt = c10::optional<torch::Tensor>;
using torch::Tensor;

std::vector<Tensor> lm_embed(Tensor tokens, Tensor table, Opt next_w,
                             double off, long n, double eps, Opt out,
                             Opt copy);
std::vector<Tensor> lm_embed_norms(Tensor tokens, Tensor table, Tensor wa,
                                   Opt wb, long n, double eps);
std::vector<Tensor> lm_add_branches(Tensor x, Opt plain, Opt o1, Opt w1,
                                    Opt o2, Opt w2, double scale, Opt wa,
                                    Opt wb, long n, double eps);
void lm_xielu(Tensor z, Tensor coef, Tensor out);
Tensor lm_post_norm_add(Tensor o, Opt bias, Tensor w, Tensor x, long n,
                        double eps, double off, Opt next_w, Opt out, Opt pos,
                        Opt share);
Tensor lm_add_norm(Tensor x, Tensor add, Opt next_w, double off, long n,
                   double eps);
Tensor lm_output_norm(Tensor x, Opt rows, Tensor w, long n, double eps,
                      double scale, double off);
Tensor lm_gated_mul(Tensor gu, Opt bias, long act);
Tensor lm_gather_rows(Tensor src, Tensor idx);
Opt lm_latent_prep(Opt q, Opt lat, Opt cq, Tensor positions, Tensor slots,
                   Tensor inv_freq, double gain, bool half, long heads,
                   long DP, long RP, long CP, long kv_rank, double eps,
                   Opt kv_norm, Opt cache, Opt q_abs, long n_abs, Opt q_norm,
                   long q_rank);
void lm_head_gemm(Tensor a, Tensor w, Tensor out, Opt gate, Opt positions,
                  Opt inv_freq, double gain, bool half, long RP);
Tensor lm_latent_attention(Tensor q_abs, Tensor cache, Tensor block_table,
                           Tensor tok_seq, Tensor positions, Opt sink,
                           double scale, long window, long CP, long max_keys);
void lm_latent_prompt(Tensor q, Tensor kv, Tensor lat, Opt sink,
                      Tensor qtiles, Tensor out, long H, long DP, long RP,
                      long CP, long VP, long window, double scale, Opt gate);
void lm_grouped_prompt(Tensor q, Tensor rows, Opt sink, Tensor qtiles,
                       Tensor out, long H, long G, long KD, long VD, bool same,
                       long window, long keep, long pool, double scale,
                       double cap, double out_scale);
void lm_grouped_prep(Tensor z, long k_at, long v_at, Tensor positions,
                     Tensor slots, Opt inv_freq, double gain, long H, long G,
                     long KD, long VD, long dim, Opt q_norm, Opt k_norm,
                     double eps, Opt first, double lam, Tensor cache, Opt bias,
                     bool whole, long pool);
void lm_grouped_pool(Tensor cache, Tensor block_table, Tensor tok_seq,
                     Tensor positions, long pool);
void lm_grouped_attention(Tensor q, Tensor cache, Tensor block_table,
                          Tensor tok_seq, Tensor positions, Opt sink,
                          Tensor out, long n, long H, long G, long KD, long VD,
                          bool same, long window, long keep, long pool,
                          double scale, double cap, double out_scale,
                          long max_keys);
void lm_linear_state(Tensor z, bool delta, long heads, long groups, long dim,
                     long vdim, long parts, double eps, Tensor conv,
                     Opt conv_b, Tensor a_log, Tensor dt_bias, Opt skip,
                     Tensor norm, Tensor state, Tensor ring, Tensor positions,
                     Tensor slots, Tensor tiles, Tensor seqs, long tile,
                     long seg, long n_single, Tensor out);
void lm_delta_rule(Tensor z, std::vector<long> at, Tensor w2, Tensor w0,
                   Tensor ab, Tensor norm, Tensor state, Tensor positions,
                   Tensor slots, Tensor seqs, Tensor out, long n_single,
                   long dim, double eps, double out_scale, long n_tiles,
                   long tile, long chunk);
std::vector<Tensor> lm_hyper_embed(Tensor tokens, Tensor table, Tensor coef,
                                   long S, long n, double eps);
Tensor lm_hyper_step(Tensor o, Tensor x, Tensor coef, long n, double eps,
                     bool last, Opt pos, Opt share, Opt skip);
Tensor lm_soft_cap(Tensor z, long n, double cap);
std::vector<Tensor> lm_moe_route(Tensor h, Tensor router, long top, long rows,
                                 bool over_all, Opt correction, long groups,
                                 long keep, long identity, long shared);
Tensor lm_moe_gemm(Tensor a, Opt tok, Tensor w, Tensor plan, long n_rows,
                   long rows, long act);
void lm_rglru_prefill(Tensor yx, Tensor byx, Tensor cw, Tensor cb, Tensor ra,
                      Tensor ba, Tensor ri, Tensor bi, Tensor lam,
                      Tensor state, Tensor ring, Tensor tiles, Tensor seqs,
                      Tensor out, long tile);
void lm_rglru_step(Tensor yx, Tensor byx, Tensor cw, Tensor cb, Tensor ra,
                   Tensor ba, Tensor ri, Tensor bi, Tensor lam, Tensor state,
                   Tensor ring, Tensor positions, Tensor slots, Tensor out,
                   long n);
Tensor skinny_gemm(Tensor a, Tensor w, int64_t variant);

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.doc() = "clearml-serving-amd gfx950 token-batch kernel library";
  m.def("lm_embed", &lm_embed);
  m.def("lm_post_norm_add", &lm_post_norm_add);
  m.def("lm_output_norm", &lm_output_norm);
  m.def("lm_add_norm", &lm_add_norm);
  m.def("lm_gated_mul", &lm_gated_mul);
  m.def("lm_gather_rows", &lm_gather_rows);
  m.def("lm_latent_prep", &lm_latent_prep);
  m.def("lm_head_gemm", &lm_head_gemm);
  m.def("lm_latent_attention", &lm_latent_attention);
  m.def("lm_latent_prompt", &lm_latent_prompt);
  m.def("lm_grouped_prompt", &lm_grouped_prompt);
  m.def("lm_grouped_prep", &lm_grouped_prep);
  m.def("lm_grouped_attention", &lm_grouped_attention);
  m.def("lm_grouped_pool", &lm_grouped_pool);
  m.def("lm_linear_state", &lm_linear_state);
  m.def("lm_embed_norms", &lm_embed_norms);
  m.def("lm_add_branches", &lm_add_branches);
  m.def("lm_xielu", &lm_xielu);
  m.def("lm_delta_rule", &lm_delta_rule);
  m.def("lm_hyper_embed", &lm_hyper_embed);
  m.def("lm_hyper_step", &lm_hyper_step);
  m.def("lm_soft_cap", &lm_soft_cap);
  m.def("lm_moe_route", &lm_moe_route);
  m.def("lm_moe_gemm", &lm_moe_gemm);
  m.def("lm_rglru_prefill", &lm_rglru_prefill);
  m.def("lm_rglru_step", &lm_rglru_step);
  m.def("skinny_gemm", &skinny_gemm, py::arg("a"), py::arg("w"),
        py::arg("variant") = 0);
}
