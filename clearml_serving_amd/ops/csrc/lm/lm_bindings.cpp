// pybind11 bindings for the token-batch kernel library (_hip_lm.so).
#include <torch/extension.h>

using Opt = c10::optional<torch::Tensor>;
using torch::Tensor;

std::vector<Tensor> lm_embed(Tensor tokens, Tensor table);
Tensor lm_post_norm_add(Tensor o, Opt bias, Tensor w, Tensor x, long n,
                        double eps);
Tensor lm_output_norm(Tensor x, Opt rows, Tensor w, long n, double eps,
                      double scale);
Tensor lm_gelu_mul(Tensor gu, Opt bias);
Tensor lm_gather_rows(Tensor src, Tensor idx);
void lm_latent_prep(Tensor qkv, Tensor positions, Tensor slots,
                    Tensor inv_freq, long heads, long DP, long RP, long CP,
                    long kv_rank, double eps, Opt kv_norm, Opt cache,
                    Opt q_abs, long n_abs);
void lm_head_gemm(Tensor a, Tensor w, Tensor out);
Tensor lm_latent_attention(Tensor q_abs, Tensor cache, Tensor block_table,
                           Tensor tok_seq, Tensor positions, Tensor sink,
                           double scale, long window, long CP, long max_keys);
void lm_latent_prompt(Tensor q, Tensor kv, Tensor lat, Tensor sink,
                      Tensor qtiles, Tensor out, long H, long DP, long RP,
                      long CP, long VP, long window, double scale);
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
  m.def("lm_gelu_mul", &lm_gelu_mul);
  m.def("lm_gather_rows", &lm_gather_rows);
  m.def("lm_latent_prep", &lm_latent_prep);
  m.def("lm_head_gemm", &lm_head_gemm);
  m.def("lm_latent_attention", &lm_latent_attention);
  m.def("lm_latent_prompt", &lm_latent_prompt);
  m.def("lm_rglru_prefill", &lm_rglru_prefill);
  m.def("lm_rglru_step", &lm_rglru_step);
  m.def("skinny_gemm", &skinny_gemm, py::arg("a"), py::arg("w"),
        py::arg("variant") = 0);
}
