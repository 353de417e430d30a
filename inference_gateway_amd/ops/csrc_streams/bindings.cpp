// Python bindings for the multi-stream decoder kernel library (gfx950):
// residual-stream steps, fixed-decay linear attention, the latent
// attention input step and expert dispatch, which are this folder's; and the
// attention, row and router kernels of csrc_hybrid and csrc_recurrent that
// such a model launches.
#include <torch/extension.h>

namespace igw {
// stream_ops.hip
int64_t stream_step_max_in_place();
void stream_step(torch::Tensor out, torch::Tensor src,
                 c10::optional<torch::Tensor> dst,
                 c10::optional<torch::Tensor> y,
                 c10::optional<torch::Tensor> mix,
                 c10::optional<torch::Tensor> outw, torch::Tensor inw,
                 torch::Tensor norm_w, double eps);
void moe_scatter_rows(torch::Tensor buf, torch::Tensor x, torch::Tensor dst,
                      int64_t K);
void moe_combine(torch::Tensor out, torch::Tensor y, torch::Tensor dst,
                 torch::Tensor w, c10::optional<torch::Tensor> shared,
                 c10::optional<torch::Tensor> g);
// latent_rope.hip
void latent_rope_append(torch::Tensor x, torch::Tensor positions,
                        torch::Tensor slot_mapping, torch::Tensor cache,
                        torch::Tensor norm_w, torch::Tensor inv_freq,
                        double eps, int64_t heads, int64_t dim,
                        int64_t rot_dim, int64_t kv_rank, bool half,
                        double mag);
// fixed_decay.hip
int64_t fixed_decay_chunk_keys();
void fixed_decay_step(torch::Tensor out, torch::Tensor q, torch::Tensor k,
                      torch::Tensor v, torch::Tensor decay,
                      torch::Tensor state, torch::Tensor seqs,
                      torch::Tensor seq_cu, torch::Tensor seq_start,
                      torch::Tensor seq_slots, bool silu);
void fixed_decay_chunks(torch::Tensor out, torch::Tensor q, torch::Tensor k,
                        torch::Tensor v, torch::Tensor decay,
                        torch::Tensor state, torch::Tensor segs,
                        c10::optional<torch::Tensor> work,
                        c10::optional<torch::Tensor> seg_first,
                        torch::Tensor seq_start, torch::Tensor seq_slots,
                        bool silu);
// csrc_hybrid: latent_attn*.hip, hybrid_ops.hip, parallel_ops.hip
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
void moe_topk_route(torch::Tensor weights, torch::Tensor idx,
                    torch::Tensor logits, c10::optional<torch::Tensor> dst,
                    c10::optional<torch::Tensor> counts, int64_t capacity,
                    double scale, bool over_all);
// csrc_recurrent: softcap_attn*.hip, qk_rope_append.hip, recurrent_ops.hip
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
void head_norm_gate(torch::Tensor out, torch::Tensor o, torch::Tensor gate,
                    torch::Tensor w, double eps, int64_t group,
                    int64_t gate_act, bool gate_first,
                    c10::optional<torch::Tensor> den,
                    c10::optional<torch::Tensor> floor_);
}  // namespace igw

PYBIND11_MODULE(TORCH_EXTENSION_NAME, m) {
  m.def("stream_step", &igw::stream_step,
        "residual streams: mix + add the sublayer's result, read off and "
        "norm the next input");
  m.def("stream_step_max_in_place", &igw::stream_step_max_in_place,
        "widest stream count that is updated in place");
  m.def("moe_scatter_rows", &igw::moe_scatter_rows,
        "token rows into the padded expert buffer");
  m.def("moe_combine", &igw::moe_combine,
        "weighted sum of expert rows plus the gated shared expert");
  m.def("latent_rope_append", &igw::latent_rope_append,
        "latent RMS norm, rotation of the shared key and the query heads, "
        "paged append");
  m.def("fixed_decay_step", &igw::fixed_decay_step,
        "fixed-decay linear attention, row by row");
  m.def("fixed_decay_chunks", &igw::fixed_decay_chunks,
        "fixed-decay linear attention on MFMA chunks (bf16)");
  m.def("fixed_decay_chunk_keys", &igw::fixed_decay_chunk_keys,
        "widest key of fixed_decay_chunks");
  m.def("gated_act", &igw::gated_act,
        "(gate | up) -> silu(g) u, the clamped gated unit or gelu_tanh(g) u");
  m.def("latent_attention", &igw::latent_attention,
        "absorbed latent attention, window, softmax sink, head gate, paged");
  m.def("latent_attention_mfma", &igw::latent_attention_mfma,
        "absorbed latent attention on MFMA tiles (bf16); false = sizes do "
        "not fit, use latent_attention");
  m.def("latent_attention_tile_rows", &igw::latent_attention_tile_rows,
        "token rows per MFMA tile for a head count");
  m.def("moe_topk_route", &igw::moe_topk_route,
        "top-k experts by logit, softmax over the chosen or over all");
  m.def("softcap_attention", &igw::softcap_attention,
        "causal paged softmax attention");
  m.def("softcap_attention_mfma", &igw::softcap_attention_mfma,
        "paged softmax attention on MFMA tiles (bf16); false = sizes do not "
        "fit, use softcap_attention");
  m.def("softcap_attention_tile_rows", &igw::softcap_attention_tile_rows,
        "query rows per MFMA tile");
  m.def("qk_norm_rope_append", &igw::qk_norm_rope_append,
        "per-head q/k RMS norm, partial pair rotation, paged K/V append");
  m.def("head_norm_gate", &igw::head_norm_gate,
        "read-out norm and output gate");
}
