// The decoder session's state, shared by the translation units that build and run one (decoder.hip: GPT-2 and Llama
// shaped layers, prompts, the generate loop; decoder_mixed.hip: layers listed one by one).
#pragma once
#include <map>
#include <string>
#include <vector>

#include "common.h"
#include "decode_fused.h"
#include "mixers.h"

namespace cthip {

struct RawTensor {
  void *dev = nullptr;  // GGUF bytes on the device
  int type = 0;
  int64_t rows = 0, cols = 0;
  size_t nbytes = 0;
};

static const int kStepsPerGraph = 8;

struct Layer {
  // GPT-2
  float *ln1_g = nullptr, *ln1_b = nullptr, *ln2_g = nullptr, *ln2_b = nullptr;
  WMat *attn = nullptr, *proj = nullptr, *fc = nullptr, *fc2 = nullptr;
  float *attn_b = nullptr, *proj_b = nullptr, *fc_b = nullptr, *fc2_b = nullptr;
  // LayerNorm folded through c_attn / c_fc: S = W.gamma, C = W.beta + bias
  float *attn_s = nullptr, *attn_c = nullptr, *fc_s = nullptr, *fc_c = nullptr;
  // Llama: attn = wq|wk|wv, proj = wo, fc = gate|up, fc2 = down, ln1_g/ln2_g = rms weights
  bool fc_pairs = false;  // gate / up rows interleaved, SwiGLU in the gate|up launch
  float *k_cache = nullptr, *v_cache = nullptr;
  // option kv_cache 1: the cache as Q8_0 rows instead (quant and scale planes; k_cache / v_cache stay null)
  void *kq = nullptr, *kdq = nullptr, *vq = nullptr, *vdq = nullptr;
  // option kv_cache 2: the cache in pages (kvp.hip): device tables of page pointers and the host's copy of them
  float **k_pages = nullptr, **v_pages = nullptr;
  std::vector<float *> k_page_host, v_page_host;
  // three-launch decode layer: attn.c_proj by head and mlp.c_proj by 16-column slab (quant / scale planes)
  void *proj_hq = nullptr, *proj_hd = nullptr, *fc2_sq = nullptr, *fc2_sd = nullptr;
};

// one mixer of a layer (decoder_mixed.hip): its rows of the layer's projection matrix start at row0, its output's columns
// of the output matrix at col0
struct MixedBranch {
  cthip_mixer_spec sp;
  std::string prefix;  // of its tensors' keys, behind "l<i>."
  int64_t row0 = 0, col0 = 0;
  WMat *absorb = nullptr, *kv_up = nullptr;  // latent: W_uk transposed per head; W_uk over W_uv
  std::vector<double> decay;                 // lightning
  // (everything but the projection rows and what a layer run keeps of the sequence)
  DeltaArgs delta = {};
  LatentArgs latent = {};
  WindowArgs window = {};
  LightningArgs lightning = {};
};
// one layer of a mixed decoder
struct MixedLayer {
  cthip_layer_spec sp;
  std::vector<MixedBranch> branches;
  float *norm1 = nullptr, *norm2 = nullptr;
  WMat *in = nullptr, *out = nullptr, *gate_up = nullptr, *down = nullptr;
  float *bias = nullptr;                   // of `in`, where a projection has one
  float *in_s = nullptr, *fc_s = nullptr;  // LayerNorm folded through `in` / `gate_up`
  float *ls1 = nullptr, *ls2 = nullptr;    // factors of the mixer's and the feed-forward's results
  bool fc_pairs = false;                   // gate / up rows interleaved, the gated unit in that launch's epilogue
  Glu glu;
  int64_t nbytes = 0;  // weights and vectors a run reads
};
// one run of a layer: looped layers run several times per token, each time with what that run has kept
struct MixedRun {
  int layer;
  bool add_embedding;      // in front of it the embedding is added to the residual stream
  float *keep[2][2] = {};  // per branch: delta ring, S; latent cache; window K, V; lightning S
};

struct Decoder {
  cthip_decoder_config cfg;
  std::map<std::string, RawTensor> raw;
  std::vector<std::string> required;
  bool finalized = false;
  std::vector<Layer> layers;
  cthip_mixed_config mcfg = {};  // arch MIXED
  std::vector<MixedLayer> mixed;
  std::vector<MixedRun> runs;
  LatentWork latent_work = {};
  ParallelWork parallel_work = {};
  float *wte = nullptr, *wpe = nullptr, *lnf_g = nullptr, *lnf_b = nullptr;
  WMat *lm_head = nullptr;
  float *lm_s = nullptr, *lm_c = nullptr;  // ln_f folded through lm_head
  // activations
  float *x = nullptr, *q = nullptr, *kv_tmp = nullptr, *att = nullptr, *h = nullptr, *logits = nullptr;
  AttnSplit att_split = {1, nullptr, nullptr};  // the one-launch-per-Linear step: workgroups per head of its attention launch
  // device-resident loop state: [0] = current token, [1] = position
  int *tokpos = nullptr;
  int64_t *token64 = nullptr;
  int64_t *history = nullptr;
  int *hist_n = nullptr;
  int *ctrl = nullptr;        // [0] = token id that ends a sequence (-1 = none), [1] = the sequence has ended
  int *ctrl_host = nullptr;   // pinned copy of ctrl the host polls between graph launches
  hipEvent_t ctrl_ev = nullptr;
  // scratch of the argmax fused behind lm_head: one partial per wavefront
  float *am_val = nullptr;
  int *am_idx = nullptr;
  int position = 0;
  bool primed = false;  // a forward has left token/position on the device
  bool use_graph = true;
  // the three-launch decode layer (decode_fused.hip): second residual buffer, per-head partials of the
  // attention projection, per-XCD accumulators of the MLP projection
  bool fused = false;
  float *x2 = nullptr, *patt = nullptr;
  long long *pmlp = nullptr;
  // all layers of a step as one launch (decode_flow.hip): the tagged hand-over buffers and the launch's arguments
  bool flow = false;
  FlowArgs flow_args = {};
  // grouped-query layers (decode_gqa.hip): the attention projection has an accumulator set of its own
  bool fused_gqa = false;
  long long *pattn = nullptr;
  // KV cache kept as Q8_0 rows (kvq.hip); peek_f32: fp32 copy of one layer's cache for cthip_decoder_peek
  bool kvq = false;
  float *peek_f32 = nullptr;
  // KV cache in pages (kvp.hip)
  bool kvp = false;
  // [0]: the step as the session runs it at short contexts; [1]: three-launch layers at long contexts (long_from > 0):
  // the attention as a launch of its own with a head's keys shared by several workgroups, then the projection
  hipGraphExec_t g_step[2] = {nullptr, nullptr}, g_body[2] = {nullptr, nullptr}, g_multi[2] = {nullptr, nullptr};
  int long_from = 0;       // position from which [1] runs; 0 = never
  bool long_mode = false;  // which of the two queue_step queues
  int64_t weight_bytes = 0, vector_bytes = 0;
  std::vector<void *> owned;  // device blocks to free
};


#define DEC_TRY(e)             \
  do {                         \
    if ((rc = (e))) return rc; \
  } while (0)

// decoder.hip
int dev_alloc(Decoder *d, void **p, size_t bytes);  // zero-filled, released with the session
int to_f32(Decoder *d, const std::string &key, int64_t want_n, float **out);
int to_wmat(Decoder *d, const std::vector<std::string> &keys, int64_t want_rows, int64_t want_cols, WMat **out, bool interleave = false);
int make_fold(Decoder *d, const WMat *w, const float *gamma, const float *beta, const float *bias, float **S, float **C);
// X += (W.in + bias) * col_scale over s rows, then XN = norm(X) with (g, b); g == nullptr: no norm follows
int linear_residual_norm(float *XN, float *X, const WMat *w, const float *in, int s, int D, const float *bias, const float *g,
                         const float *b, float eps, bool rms, int precision, const float *col_scale = nullptr);
// decoder_mixed.hip
void mixed_required(Decoder *d);
int mixed_load(Decoder *d);              // the layers' matrices, states and caches out of the loaded tensors
void mixed_release(Decoder *d);
int mixed_queue_layers(Decoder *d);      // one decode step's layers, d->x in place
int mixed_prefill(Decoder *d, float *X, float *XN, const int *ids, int s, int n);  // s rows at positions n .., X in place
int mixed_launches(const Decoder *d);    // the most launches any layer runs in a decode step
int64_t mixed_state_bytes(const Decoder *d, int t);  // cache and state bytes of a step at position t
int mixed_peek(Decoder *d, const char *what, void **ptr, int64_t *n_floats);  // 1 = not one of its buffers

}  // namespace cthip
