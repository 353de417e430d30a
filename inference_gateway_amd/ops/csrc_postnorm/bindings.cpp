// Python bindings for the post-norm decoder kernel library (gfx950):
// windowed softmax attention over paged keys and values, latent attention,
// the row kernels around them and the gated feed-forward.  Every kernel is
// a source file of csrc_hybrid or csrc_recurrent; this extension links just
// the ones such a model launches, so serving it compiles and loads nothing
// else.
#include <torch/extension.h>

namespace igw {
// csrc_hybrid: latent_attn*.hip, hybrid_ops.hip, parallel_ops.hip
void latent_down_post(torch::Tensor cq, torch::Tensor gate, torch::Tensor down,
                      torch::Tensor positions, torch::Tensor slot_mapping,
                      c10::optional<torch::Tensor> cache,
                      torch::Tensor qnorm_w,
                      c10::optional<torch::Tensor> kvnorm_w,
                      torch::Tensor inv_freq, double eps, int64_t q_rank,
                      int64_t kv_rank, int64_t rot_dim, int64_t heads,
                      bool half, double mag);
void rope_pairs(torch::Tensor x, torch::Tensor positions,
                torch::Tensor inv_freq, int64_t offset, bool half,
                double mag);
void gated_act(torch::Tensor out, torch::Tensor in, int64_t mode, double limit,
               double alpha);
void latent_attention(torch::Tensor out, torch::Tensor q_abs,
                      torch::Tensor q_rot, torch::Tensor cache,
                      torch::Tensor block_table, torch::Tensor row_seq,
                      torch::Tensor positions,
                      c10::optional<torch::Tensor> sink, double scale,
                      int64_t window, c10::optional<torch::Tensor> gate);
bool latent_attention_mfma(torch::Tensor out, torch::Tensor q_abs,
                           torch::Tensor q_rot, torch::Tensor cache,
                           torch::Tensor block_table, torch::Tensor row_seq,
                           torch::Tensor positions, torch::Tensor tile_row0,
                           torch::Tensor tile_nrows,
                           c10::optional<torch::Tensor> sink, double scale,
                           int64_t window, int64_t max_keys,
                           c10::optional<torch::Tensor> gate);
int64_t latent_attention_tile_rows(int64_t H);
// csrc_recurrent: softcap_attn*.hip, qk_rope_append.hip, sandwich_ops.hip
void softcap_attention(torch::Tensor out, torch::Tensor q, torch::Tensor kcache,
                       torch::Tensor vcache, torch::Tensor block_table,
                       torch::Tensor row_seq, torch::Tensor positions,
                       double scale, double softcap, double temp_coef,
                       int64_t temp_every, int64_t window,
                       c10::optional<torch::Tensor> slopes, int64_t chunk,
                       c10::optional<torch::Tensor> sinks,
                       c10::optional<torch::Tensor> gate, int64_t keep);
bool softcap_attention_mfma(torch::Tensor out, torch::Tensor q,
                            torch::Tensor kcache, torch::Tensor vcache,
                            torch::Tensor block_table, torch::Tensor seq_cu,
                            torch::Tensor seq_start, torch::Tensor tile_seq,
                            torch::Tensor tile_off, torch::Tensor dec_seq,
                            double scale, double softcap, double temp_coef,
                            int64_t temp_every, int64_t window,
                            c10::optional<torch::Tensor> slopes,
                            int64_t chunk, c10::optional<torch::Tensor> sinks,
                            c10::optional<torch::Tensor> gate, int64_t keep);
int64_t softcap_attention_tile_rows();
void qk_norm_rope_append(torch::Tensor qout, torch::Tensor proj,
                         torch::Tensor positions, torch::Tensor slot_mapping,
                         torch::Tensor kcache, torch::Tensor vcache,
                         c10::optional<torch::Tensor> qnorm_w,
                         c10::optional<torch::Tensor> knorm_w,
                         c10::optional<torch::Tensor> inv_freq, double mag,
                         double eps, int64_t heads, int64_t kv_heads,
                         int64_t dim, int64_t vdim, bool half,
                         bool tied);
void add_normed_rmsnorm(torch::Tensor out, torch::Tensor residual,
                        c10::optional<torch::Tensor> delta,
                        c10::optional<torch::Tensor> w_post,
                        c10::optional<torch::Tensor> w_pre, double eps,
                        double mult);
}  // namespace igw

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("latent_down_post", &igw::latent_down_post,
        "latent RMS norms + shared-key rotation + paged append + head gates");
  m.def("rope_pairs", &igw::rope_pairs,
        "in-place rotary on a slice of every head, interleaved or half pairs");
  m.def("gated_act", &igw::gated_act,
        "(gate | up) -> silu(g) u, the clamped gated unit or gelu_tanh(g) u");
  m.def("latent_attention", &igw::latent_attention,
        "absorbed latent attention, window, softmax sink, head gate, paged");
  m.def("latent_attention_mfma", &igw::latent_attention_mfma,
        "absorbed latent attention on MFMA tiles (bf16); false = sizes do "
        "not fit, use latent_attention");
  m.def("latent_attention_tile_rows", &igw::latent_attention_tile_rows,
        "token rows per MFMA tile for a head count");
  m.def("softcap_attention", &igw::softcap_attention,
        "causal paged softmax attention with a tanh score cap");
  m.def("softcap_attention_mfma", &igw::softcap_attention_mfma,
        "capped softmax attention on MFMA tiles (bf16); false = sizes do "
        "not fit, use softcap_attention");
  m.def("softcap_attention_tile_rows", &igw::softcap_attention_tile_rows,
        "query rows per MFMA tile");
  m.def("qk_norm_rope_append", &igw::qk_norm_rope_append,
        "per-head q/k RMS norm, partial pair rotation, paged K/V append");
  m.def("add_normed_rmsnorm", &igw::add_normed_rmsnorm,
        "fp32 residual += scaled RMS-normed delta; RMS norm of the sum");
}
