// Layers of a mixed decoder (cthip_decoder_create_mixed): each has a token mixer of its own kind and sizes and an
// optional SwiGLU feed-forward.  Not in the reference, whose Transformer repeats one block
// (external/llm/layers.lisp:73-90); embedding, head, prompts, graphs and the generate loop are decoder.hip's.
//
// All projections that read norm1(x) are one matrix, so a decode step is, per layer:
//   delta    norm1 -> [q k v g b a] GEMV;  k_delta_step;  o GEMV + residual
//   latent   norm1 -> [q latent g] GEMV;  k_latent_absorb, _attend, _up;  o GEMV + residual
//   ff       norm2 -> gate|up GEMV (SwiGLU in its epilogue where a launch holds row pairs);  down GEMV + residual
// Head sizes are padded to multiples of 16 when the matrices are put together (mixers.h).
#include <string.h>

#include <algorithm>

#include "decoder.h"

namespace cthip {

static std::string mkey(int l, const char *s) { return "l" + std::to_string(l) + "." + s; }

void mixed_required(Decoder *d) {
  d->required = {"embed", "final.norm", "head"};
  for (int l = 0; l < d->cfg.n_layers; l++) {
    const cthip_layer_spec &sp = d->mixed[l].sp;
    std::vector<const char *> keys = {"norm1", "mix.q", "mix.o"};
    if (sp.mixer == CTHIP_MIXER_DELTA)
      keys.insert(keys.end(), {"mix.q.conv", "mix.k", "mix.k.conv", "mix.v", "mix.v.conv", "mix.b", "mix.a", "mix.A_log", "mix.dt_bias",
                               "mix.g", "mix.norm"});
    else {
      keys.insert(keys.end(), {"mix.dkv", "mix.dkv.norm", "mix.uk", "mix.uv"});
      if (sp.sink) keys.push_back("mix.sink");
      if (sp.gate) keys.push_back("mix.g");
    }
    if (sp.ffn) keys.insert(keys.end(), {"norm2", "mlp.gate", "mlp.up", "mlp.down"});
    for (const char *k : keys) d->required.push_back(mkey(l, k));
  }
}

// a loaded tensor of the given shape
static int raw_of(Decoder *d, const std::string &key, int64_t rows, int64_t cols, RawTensor **out) {
  auto it = d->raw.find(key);
  if (it == d->raw.end()) return fail(CTHIP_E_STATE, "decoder: tensor '%s' was not loaded", key.c_str());
  RawTensor &r = it->second;
  if (r.rows != rows || r.cols != cols)
    return fail(CTHIP_E_BAD_ARG, "decoder: tensor '%s' is (%lld,%lld), expected (%lld,%lld)", key.c_str(), (long long)r.rows, (long long)r.cols,
                (long long)rows, (long long)cols);
  *out = &r;
  return 0;
}

// an all-zero weight matrix to place parts in
static int wmat_empty(Decoder *d, int type, int64_t rows, int64_t cols, WMat **out) {
  if (type != CTHIP_F32 && type != CTHIP_F16 && type != CTHIP_BF16)
    return fail(CTHIP_E_UNSUPPORTED, "decoder: the Linear weights of a mixed decoder are fp32, fp16 or bf16, not ggml type %d", type);
  WMat *w = new WMat();
  w->type = type;
  w->rows = rows;
  w->cols = cols;
  w->d = nullptr;
  w->d_bytes = 0;
  w->q_bytes = rows * cols * (type == CTHIP_F32 ? 4 : 2);
  const int rc = cthip_alloc(&w->q, (size_t)w->q_bytes);  // zero-filled
  if (rc) {
    delete w;
    return rc;
  }
  w->stream = w->q_bytes > kInfinityCacheBytes;
  d->weight_bytes += w->q_bytes;
  if (!gemv_is_direct(w)) d->use_graph = false;
  *out = w;
  return 0;
}
static int elem(const WMat *w) { return w->type == CTHIP_F32 ? 4 : 2; }

// rows of a loaded (rows, w->cols) tensor in heads of hr, placed from row r0 on, hrp apart
static int place_rows(Decoder *d, WMat *w, const std::string &key, int64_t rows, int64_t r0, int64_t hr, int64_t hrp, int64_t cols = 0) {
  RawTensor *r = nullptr;
  const int64_t n = cols ? cols : w->cols;
  int rc = raw_of(d, key, rows, n, &r);
  if (rc) return rc;
  if (r->type != w->type) return fail(CTHIP_E_BAD_ARG, "decoder: tensor '%s' has ggml type %d, its neighbours %d", key.c_str(), r->type, w->type);
  return launch_place(w->q, r->dev, elem(w), rows, n, r0, hr, hrp, n, n, w->cols);
}

// fp32 vector of a tensor of n elements in heads of hr, hrp apart in the padded vector
static int vec_padded(Decoder *d, const std::string &key, int64_t n, int64_t hr, int64_t hrp, float **out) {
  float *tmp = nullptr;
  int rc = to_f32(d, key, n, &tmp);
  if (rc) return rc;
  if (hr == hrp) {
    *out = tmp;
    return 0;
  }
  if ((rc = dev_alloc(d, (void **)out, sizeof(float) * (size_t)(n / hr * hrp)))) return rc;
  return launch_place(*out, tmp, 4, n, 1, 0, hr, hrp, 1, 1, 1);
}

static int load_delta(Decoder *d, int l) {
  MixedLayer &L = d->mixed[l];
  const cthip_layer_spec &sp = L.sp;
  const int D = d->cfg.dim, H = sp.heads, KH = sp.kv_heads, dk = sp.dim, dv = sp.vdim;
  DeltaArgs &a = L.delta;
  a.H = H, a.KH = KH, a.dk = dk, a.dv = dv, a.DK = pad16(dk), a.DV = pad16(dv), a.taps = sp.conv;
  const int KQ = KH * a.DK, VW = H * a.DV, C = a.C = 2 * KQ + VW;
  a.ldp = pad16(C + VW + 2 * H);
  a.eps = d->cfg.eps;
  int rc;
  RawTensor *q = nullptr;
  DEC_TRY(raw_of(d, mkey(l, "mix.q"), (int64_t)KH * dk, D, &q));
  DEC_TRY(wmat_empty(d, q->type, a.ldp, D, &L.in));
  DEC_TRY(place_rows(d, L.in, mkey(l, "mix.q"), (int64_t)KH * dk, 0, dk, a.DK));
  DEC_TRY(place_rows(d, L.in, mkey(l, "mix.k"), (int64_t)KH * dk, KQ, dk, a.DK));
  DEC_TRY(place_rows(d, L.in, mkey(l, "mix.v"), (int64_t)H * dv, 2 * KQ, dv, a.DV));
  DEC_TRY(place_rows(d, L.in, mkey(l, "mix.g"), (int64_t)H * dv, C, dv, a.DV));
  DEC_TRY(place_rows(d, L.in, mkey(l, "mix.b"), H, C + VW, H, H));
  DEC_TRY(place_rows(d, L.in, mkey(l, "mix.a"), H, C + VW + H, H, H));
  float *conv = nullptr, *taps = nullptr, *alog = nullptr, *na = nullptr, *v = nullptr;
  DEC_TRY(dev_alloc(d, (void **)&conv, sizeof(float) * (size_t)a.taps * C));
  struct { const char *key; int channels, ch0, hr, hrp; } parts[] = {
      {"mix.q.conv", KH * dk, 0, dk, a.DK}, {"mix.k.conv", KH * dk, KQ, dk, a.DK}, {"mix.v.conv", H * dv, 2 * KQ, dv, a.DV}};
  for (auto &p : parts) {
    RawTensor *r = nullptr;
    DEC_TRY(raw_of(d, mkey(l, p.key), p.channels, a.taps, &r));
    DEC_TRY(to_f32(d, mkey(l, p.key), (int64_t)p.channels * a.taps, &taps));
    DEC_TRY(launch_place_taps(conv, taps, p.channels, a.taps, C, p.ch0, p.hr, p.hrp));
  }
  a.conv = conv;
  DEC_TRY(to_f32(d, mkey(l, "mix.A_log"), H, &alog));
  DEC_TRY(dev_alloc(d, (void **)&na, sizeof(float) * (size_t)H));
  DEC_TRY(launch_neg_exp(na, alog, H));
  a.neg_a = na;
  DEC_TRY(to_f32(d, mkey(l, "mix.dt_bias"), H, &v));
  a.dt_bias = v;
  DEC_TRY(vec_padded(d, mkey(l, "mix.norm"), dv, dv, a.DV, &v));
  a.norm = v;
  // the sequence's state: the recurrence's matrices and the convolutions' last inputs
  DEC_TRY(dev_alloc(d, (void **)&a.ring, sizeof(float) * (size_t)a.taps * C));
  DEC_TRY(dev_alloc(d, (void **)&a.S, sizeof(float) * (size_t)H * a.DV * a.DK));
  return 0;
}

static int load_latent(Decoder *d, int l) {
  MixedLayer &L = d->mixed[l];
  const cthip_layer_spec &sp = L.sp;
  const int D = d->cfg.dim, H = sp.heads, dk = sp.dim, dv = sp.vdim, r = sp.kv_rank;
  LatentArgs &a = L.latent;
  a.H = H, a.dk = dk, a.dv = dv, a.r = r, a.DK = pad16(dk), a.DV = pad16(dv), a.R = pad16(r);
  a.ldp = (int64_t)H * a.DK + a.R + (sp.gate ? H * a.DV : 0);
  a.eps = d->cfg.eps;
  a.scale = sp.scale;
  a.gated = sp.gate;
  int rc;
  RawTensor *q = nullptr, *uk = nullptr;
  DEC_TRY(raw_of(d, mkey(l, "mix.q"), (int64_t)H * dk, D, &q));
  DEC_TRY(wmat_empty(d, q->type, a.ldp, D, &L.in));
  DEC_TRY(place_rows(d, L.in, mkey(l, "mix.q"), (int64_t)H * dk, 0, dk, a.DK));
  DEC_TRY(place_rows(d, L.in, mkey(l, "mix.dkv"), r, (int64_t)H * a.DK, r, r));
  if (sp.gate) DEC_TRY(place_rows(d, L.in, mkey(l, "mix.g"), (int64_t)H * dv, (int64_t)H * a.DK + a.R, dv, a.DV));
  DEC_TRY(raw_of(d, mkey(l, "mix.uk"), (int64_t)H * dk, r, &uk));
  if (uk->type != q->type) return fail(CTHIP_E_BAD_ARG, "decoder: '%s' has ggml type %d, the layer's other weights %d", mkey(l, "mix.uk").c_str(), uk->type, q->type);
  DEC_TRY(wmat_empty(d, uk->type, (int64_t)H * a.R, a.DK, &L.absorb));
  DEC_TRY(launch_place_transposed(L.absorb->q, uk->dev, elem(L.absorb), H, dk, a.DK, r, a.R));
  DEC_TRY(wmat_empty(d, uk->type, (int64_t)H * (a.DK + a.DV), a.R, &L.kv_up));
  d->weight_bytes -= (int64_t)H * a.DK * a.R * elem(L.kv_up);  // (a decode step reads the key projection from `absorb` only)
  DEC_TRY(place_rows(d, L.kv_up, mkey(l, "mix.uk"), (int64_t)H * dk, 0, dk, a.DK, r));
  DEC_TRY(place_rows(d, L.kv_up, mkey(l, "mix.uv"), (int64_t)H * dv, (int64_t)H * a.DK, dv, a.DV, r));
  a.type = uk->type;
  a.absorb = L.absorb->q;
  a.up = (const char *)L.kv_up->q + (int64_t)H * a.DK * a.R * elem(L.kv_up);
  float *v = nullptr;
  DEC_TRY(vec_padded(d, mkey(l, "mix.dkv.norm"), r, r, a.R, &v));
  a.norm = v;
  if (sp.sink) {
    DEC_TRY(to_f32(d, mkey(l, "mix.sink"), H, &v));
    a.sink = v;
  }
  a.rows = d->cfg.max_seq;
  DEC_TRY(dev_alloc(d, (void **)&a.cache, sizeof(float) * (size_t)a.rows * a.R));
  return 0;
}

int mixed_load(Decoder *d) {
  const cthip_decoder_config &c = d->cfg;
  const cthip_mixed_config &mc = d->mcfg;
  const int D = c.dim, V = c.vocab;
  const bool ln = mc.norm == CTHIP_PRO_LAYERNORM;
  int rc;
  DEC_TRY(to_f32(d, "embed", (int64_t)V * D, &d->wte));
  if (mc.position_base > 0.0f) {
    DEC_TRY(dev_alloc(d, (void **)&d->wpe, sizeof(float) * (size_t)c.max_seq * D));
    DEC_TRY(launch_sinusoid_table(d->wpe, c.max_seq, D, mc.position_base));
  }
  DEC_TRY(to_f32(d, "final.norm", D, &d->lnf_g));
  DEC_TRY(to_wmat(d, {"head"}, V, D, &d->lm_head));
  float *none = nullptr;
  if (ln) DEC_TRY(make_fold(d, d->lm_head, d->lnf_g, nullptr, nullptr, &d->lm_s, &none));
  int64_t most_p = 0, most_o = 0, most_h = 0, most_qa = 0, most_part = 0;
  for (int l = 0; l < c.n_layers; l++) {
    MixedLayer &L = d->mixed[l];
    const cthip_layer_spec &sp = L.sp;
    const bool delta = sp.mixer == CTHIP_MIXER_DELTA;
    DEC_TRY(to_f32(d, mkey(l, "norm1"), D, &L.norm1));
    DEC_TRY(delta ? load_delta(d, l) : load_latent(d, l));
    if (ln) DEC_TRY(make_fold(d, L.in, L.norm1, nullptr, nullptr, &L.in_s, &none));
    const int DV = pad16(sp.vdim), H = sp.heads;
    RawTensor *o = nullptr;
    DEC_TRY(raw_of(d, mkey(l, "mix.o"), D, (int64_t)H * sp.vdim, &o));
    DEC_TRY(wmat_empty(d, o->type, D, (int64_t)H * DV, &L.out));
    DEC_TRY(launch_place(L.out->q, o->dev, elem(L.out), D, (int64_t)H * sp.vdim, 0, D, D, sp.vdim, DV, (int64_t)H * DV));
    if (sp.ffn) {
      DEC_TRY(to_f32(d, mkey(l, "norm2"), D, &L.norm2));
      RawTensor *g = nullptr;
      DEC_TRY(raw_of(d, mkey(l, "mlp.gate"), sp.ffn, D, &g));
      L.fc_pairs = gemv_pair_swiglu_ok(g->type, 2 * (int64_t)sp.ffn, D, ln);
      DEC_TRY(to_wmat(d, {mkey(l, "mlp.gate"), mkey(l, "mlp.up")}, 2 * (int64_t)sp.ffn, D, &L.gate_up, L.fc_pairs));
      DEC_TRY(to_wmat(d, {mkey(l, "mlp.down")}, D, sp.ffn, &L.down));
      if (ln) DEC_TRY(make_fold(d, L.gate_up, L.norm2, nullptr, nullptr, &L.fc_s, &none));
    }
    most_p = std::max(most_p, delta ? L.delta.ldp : L.latent.ldp);
    most_o = std::max(most_o, (int64_t)H * DV);
    most_h = std::max(most_h, 2 * (int64_t)sp.ffn);
    if (!delta) {
      // key ranges of the decode attention: as many workgroups as there are compute units, at least a tile each
      int ranges = state().compute_units / ((H + 15) / 16);
      ranges = std::min({ranges, kLatentMaxRanges, (c.max_seq + 15) / 16});
      d->latent_work.ranges = d->latent_work.ranges ? std::min(d->latent_work.ranges, std::max(ranges, 1)) : std::max(ranges, 1);
      most_qa = std::max(most_qa, (int64_t)H * L.latent.R);
      most_part = std::max(most_part, (int64_t)latent_part_floats(H, L.latent.R, kLatentMaxRanges));
    }
  }
  DEC_TRY(dev_alloc(d, (void **)&d->q, sizeof(float) * (size_t)most_p));
  DEC_TRY(dev_alloc(d, (void **)&d->att, sizeof(float) * (size_t)most_o));
  if (most_h) DEC_TRY(dev_alloc(d, (void **)&d->h, sizeof(float) * (size_t)most_h));
  if (most_qa) {
    DEC_TRY(dev_alloc(d, (void **)&d->latent_work.qa, sizeof(float) * (size_t)most_qa));
    DEC_TRY(dev_alloc(d, (void **)&d->latent_work.part, sizeof(float) * (size_t)most_part));
  }
  return 0;
}

void mixed_release(Decoder *d) {
  for (MixedLayer &L : d->mixed)
    for (WMat *w : {L.in, L.out, L.gate_up, L.down, L.absorb, L.kv_up}) cthip_wmat_destroy(w);
}

int mixed_launches(const Decoder *d) {
  int most = 0;
  for (const MixedLayer &L : d->mixed) most = std::max(most, (L.sp.mixer == CTHIP_MIXER_DELTA ? 3 : 5) + (L.sp.ffn ? 2 : 0));
  return most;
}

int64_t mixed_state_bytes(const Decoder *d, int t) {
  int64_t n = 0;
  for (const MixedLayer &L : d->mixed) {
    if (L.sp.mixer == CTHIP_MIXER_DELTA) n += 4 * (2ll * L.delta.H * L.delta.DV * L.delta.DK + (int64_t)L.delta.taps * L.delta.C);
    else n += 4 * (int64_t)(t + 1) * L.latent.R;
  }
  return n;
}

int mixed_peek(Decoder *d, const char *what, void **ptr, int64_t *n_floats) {
  int l = -1;
  int64_t n = 0;
  if (sscanf(what, "latent.%d", &l) == 1 && l >= 0 && l < d->cfg.n_layers && d->mixed[l].sp.mixer == CTHIP_MIXER_LATENT) {
    *ptr = d->mixed[l].latent.cache;
    n = (int64_t)d->cfg.max_seq * d->mixed[l].latent.R;
  } else if (sscanf(what, "state.%d", &l) == 1 && l >= 0 && l < d->cfg.n_layers && d->mixed[l].sp.mixer == CTHIP_MIXER_DELTA) {
    const DeltaArgs &a = d->mixed[l].delta;
    *ptr = a.S;
    n = (int64_t)a.H * a.DV * a.DK;
  } else {
    return 1;
  }
  if (n_floats) *n_floats = n;
  return 0;
}

int mixed_queue_layers(Decoder *d) {
  const int D = d->cfg.dim, pro = d->mcfg.norm;
  const int *pos = d->tokpos + 1;
  int rc;
  auto normed = [&](const WMat *w, const float *g, const float *fold, float *y, bool pairs) {
    GemvArgs a = {};
    a.x = d->x;
    a.pro = pro;
    a.norm_g = g;
    a.eps = d->cfg.eps;
    a.fold_s = fold;
    a.pair_swiglu = pairs ? 1 : 0;
    a.y = y;
    a.x_stride = D;
    a.y_stride = pairs ? w->rows / 2 : w->rows;
    return launch_gemv(w, a, 1);
  };
  auto residual = [&](const WMat *w, const float *x, int xpro) {
    GemvArgs a = {};
    a.x = x;
    a.pro = xpro;
    a.residual = d->x;
    a.y = d->x;
    a.x_stride = xpro == CTHIP_PRO_SWIGLU ? 2 * w->cols : w->cols;
    a.y_stride = D;
    return launch_gemv(w, a, 1);
  };
  for (MixedLayer &L : d->mixed) {
    DEC_TRY(normed(L.in, L.norm1, L.in_s, d->q, false));
    if (L.sp.mixer == CTHIP_MIXER_DELTA) {
      DeltaArgs a = L.delta;
      a.p = d->q;
      DEC_TRY(launch_delta_step(a, d->att, d->tokpos, d->ctrl));
    } else {
      LatentArgs a = L.latent;
      a.p = d->q;
      DEC_TRY(launch_latent_step(a, d->latent_work, d->att, pos));
    }
    DEC_TRY(residual(L.out, d->att, CTHIP_PRO_NONE));
    if (L.sp.ffn) {
      DEC_TRY(normed(L.gate_up, L.norm2, L.fc_s, d->h, L.fc_pairs));
      DEC_TRY(residual(L.down, d->h, L.fc_pairs ? CTHIP_PRO_NONE : CTHIP_PRO_SWIGLU));
    }
  }
  return 0;
}

int mixed_prefill(Decoder *d, float *X, float *XN, int s, int n) {
  const cthip_decoder_config &c = d->cfg;
  const int D = c.dim;
  const bool rms = d->mcfg.norm == CTHIP_PRO_RMSNORM;
  const int prec = d->mcfg.precision >= 0 ? d->mcfg.precision : state().gemm_precision;
  size_t most_p = 0, most_o = 0, most_h = 0, most_g = 0, most_w = 0;
  for (const MixedLayer &L : d->mixed) {
    const bool delta = L.sp.mixer == CTHIP_MIXER_DELTA;
    most_p = std::max(most_p, (size_t)s * L.in->rows);
    most_o = std::max(most_o, (size_t)s * L.out->cols);
    most_w = std::max(most_w, delta ? delta_scratch_floats(L.delta, s) : (size_t)(n + s) * L.kv_up->rows);
    if (L.sp.ffn) most_h = std::max(most_h, (size_t)s * 2 * L.sp.ffn), most_g = std::max(most_g, (size_t)s * L.sp.ffn);
  }
  float *P = nullptr, *O = nullptr, *Hb = nullptr, *G = nullptr, *W = nullptr;
  int rc = 0;
  auto run = [&]() -> int {
    int rc;
    DEC_TRY(alloc_scratch((void **)&P, sizeof(float) * most_p));
    DEC_TRY(alloc_scratch((void **)&O, sizeof(float) * most_o));
    DEC_TRY(alloc_scratch((void **)&W, sizeof(float) * most_w));
    if (most_h) {
      DEC_TRY(alloc_scratch((void **)&Hb, sizeof(float) * most_h));
      DEC_TRY(alloc_scratch((void **)&G, sizeof(float) * most_g));
    }
    DEC_TRY(rms ? cthip_rmsnorm(XN, X, d->mixed[0].norm1, c.eps, s, D) : cthip_layernorm(XN, X, d->mixed[0].norm1, nullptr, c.eps, s, D));
    for (int l = 0; l < c.n_layers; l++) {
      MixedLayer &L = d->mixed[l];
      DEC_TRY(launch_linear_gemm(P, L.in, XN, s, nullptr, nullptr, CTHIP_ACT_NONE, prec));
      if (L.sp.mixer == CTHIP_MIXER_DELTA) {
        DeltaArgs a = L.delta;
        a.p = P;
        DEC_TRY(launch_delta_rows(a, O, s, n, W));
      } else {
        LatentArgs a = L.latent;
        a.p = P;
        DEC_TRY(launch_latent_append(a, s, n));
        // keys and values of every visible row
        DEC_TRY(launch_linear_gemm(W, L.kv_up, a.cache, n + s, nullptr, nullptr, CTHIP_ACT_NONE, prec));
        AttnRowsArgs r = {};
        r.out = O;
        r.q = P;
        r.k = W;
        r.v = W + (size_t)a.H * a.DK;
        r.S = s;
        r.start_pos = n;
        r.H = r.Hkv = a.H;
        r.ldq = r.ldg = (int)a.ldp;
        r.ldk = r.ldv = (int)L.kv_up->rows;
        r.ldo = (int)L.out->cols;
        r.dk = a.DK;
        r.dv = a.DV;
        r.scale = a.scale;
        r.sink = a.sink;
        r.gate = a.gated ? P + (size_t)a.H * a.DK + a.R : nullptr;
        DEC_TRY(launch_attn_rows(r, prec == GEMM_FP32));
      }
      const float *next = l + 1 < c.n_layers ? d->mixed[l + 1].norm1 : nullptr;
      DEC_TRY(linear_residual_norm(XN, X, L.out, O, s, D, nullptr, L.sp.ffn ? L.norm2 : next, nullptr, c.eps, rms, prec));
      if (L.sp.ffn) {
        const int F = L.sp.ffn;
        if (L.fc_pairs && (2 * F) % 4 == 0) {
          DEC_TRY(launch_linear_gemm(G, L.gate_up, XN, s, nullptr, nullptr, kActSwigluPairs, prec));
        } else {
          DEC_TRY(launch_linear_gemm(Hb, L.gate_up, XN, s, nullptr, nullptr, CTHIP_ACT_NONE, prec));
          if (L.fc_pairs) DEC_TRY(launch_swiglu_pairs(G, Hb, (int64_t)s * F));
          else DEC_TRY(launch_prologue(G, Hb, F, CTHIP_PRO_SWIGLU, nullptr, nullptr, 0.0f, 2 * (int64_t)F, s));
        }
        DEC_TRY(linear_residual_norm(XN, X, L.down, G, s, D, nullptr, next, nullptr, c.eps, rms, prec));
      }
    }
    return 0;
  };
  rc = run();
  for (void *p : {(void *)P, (void *)O, (void *)Hb, (void *)G, (void *)W})
    if (p) cthip_free(p);
  return rc;
}

}  // namespace cthip
