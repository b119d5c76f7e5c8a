// Layers of a mixed decoder (cthip_decoder_create_mixed): each has a token mixer of its own kind and sizes, or two side by
// side, and an optional gated feed-forward; some layers may run several times per token.  Not in the reference, whose
// Transformer repeats one block (external/llm/layers.lisp:73-90); embedding, head, prompts, graphs and the generate loop
// are decoder.hip's.
//
// All projections that read norm1(x) are one matrix, so a decode step is, per layer run:
//   delta              norm1 -> [q k v g b a] GEMV;  k_delta_step;  o GEMV + residual
//   latent             norm1 -> [q latent g] GEMV;  k_latent_absorb, _attend, _up;  o GEMV + residual
//   window, lightning  norm1 -> [q k v g] GEMV (of both);  k_parallel_step (both);  [o o] GEMV + residual
//   ff                 norm2 -> gate|up GEMV (the gated unit in its epilogue where a launch holds row pairs);  down GEMV + residual
// Head sizes are padded to multiples of 16 when the matrices are put together (mixers.h).
#include <string.h>

#include <math.h>

#include <algorithm>
#include <map>
#include <tuple>

#include "decoder.h"

namespace cthip {

static std::string mkey(int l, const std::string &s) { return "l" + std::to_string(l) + "." + s; }

void mixed_required(Decoder *d) {
  d->required = {"embed", "final.norm"};
  if (!d->mcfg.tied_head) d->required.push_back("head");
  for (int l = 0; l < d->cfg.n_layers; l++) {
    const MixedLayer &L = d->mixed[l];
    std::vector<std::string> keys = {"norm1"};
    for (const MixedBranch &br : L.branches) {
      const cthip_mixer_spec &sp = br.sp;
      std::vector<const char *> own = {"q", "o"};
      if (sp.mixer == CTHIP_MIXER_DELTA) {
        own.insert(own.end(), {"q.conv", "k", "k.conv", "v", "v.conv", "b", "a", "A_log", "dt_bias", "g", "norm"});
      } else if (sp.mixer == CTHIP_MIXER_LATENT) {
        own.insert(own.end(), {"dkv", "dkv.norm", "uk", "uv"});
      } else if (sp.mixer == CTHIP_MIXER_LIGHTNING) {
        own.insert(own.end(), {"k", "v", "g", "norm"});
      } else {
        own.insert(own.end(), {"k", "v"});
        if (sp.bias) own.insert(own.end(), {"q.b", "k.b", "v.b"});
        if (sp.qk_norm) own.insert(own.end(), {"q.norm", "k.norm"});
      }
      if (sp.mixer == CTHIP_MIXER_LATENT || sp.mixer == CTHIP_MIXER_WINDOW) {
        if (sp.sink == CTHIP_SINK_TENSOR) own.push_back("sink");
        if (sp.gate) own.push_back("g");
      }
      for (const char *k : own) keys.push_back(br.prefix + k);
    }
    if (L.sp.layer_scale) keys.push_back("ls1");
    if (L.sp.ffn) {
      keys.insert(keys.end(), {"norm2", "mlp.gate", "mlp.up", "mlp.down"});
      if (L.sp.layer_scale) keys.push_back("ls2");
    }
    for (const std::string &k : keys) d->required.push_back(mkey(l, k));
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

// The projection matrix of a layer: `rows` of it, of the type of its first branch's queries.  Branches place their rows in it.
static int in_matrix(Decoder *d, int l, int64_t rows) {
  MixedLayer &L = d->mixed[l];
  const std::string key = mkey(l, L.branches[0].prefix + "q");
  auto it = d->raw.find(key);
  if (it == d->raw.end()) return fail(CTHIP_E_STATE, "decoder: tensor '%s' was not loaded", key.c_str());
  return wmat_empty(d, it->second.type, rows, d->cfg.dim, &L.in);
}
// rows of the projection matrix that a branch takes
static int64_t branch_rows(const cthip_mixer_spec &sp) {
  const int64_t H = sp.heads, G = sp.kv_heads, DK = pad16(sp.dim), DV = pad16(sp.vdim);
  switch (sp.mixer) {
    case CTHIP_MIXER_DELTA: return pad16(2 * G * DK + 2 * H * DV + 2 * H);
    case CTHIP_MIXER_LATENT: return H * DK + pad16(sp.kv_rank) + (sp.gate ? H * DV : 0);
    case CTHIP_MIXER_WINDOW: return H * DK + G * (DK + DV) + (sp.gate ? H * DV : 0);
    default: return 2 * H * (DK + DV);
  }
}

static int load_delta(Decoder *d, int l, MixedBranch &br) {
  MixedLayer &L = d->mixed[l];
  const cthip_mixer_spec &sp = br.sp;
  const int H = sp.heads, KH = sp.kv_heads, dk = sp.dim, dv = sp.vdim;
  auto key = [&](const char *k) { return mkey(l, br.prefix + k); };
  DeltaArgs &a = br.delta;
  a.H = H, a.KH = KH, a.dk = dk, a.dv = dv, a.DK = pad16(dk), a.DV = pad16(dv), a.taps = sp.conv;
  const int KQ = KH * a.DK, VW = H * a.DV, C = a.C = 2 * KQ + VW;
  const int64_t r0 = br.row0;
  a.ldp = L.in->rows;
  a.eps = d->cfg.eps;
  int rc;
  DEC_TRY(place_rows(d, L.in, key("q"), (int64_t)KH * dk, r0, dk, a.DK));
  DEC_TRY(place_rows(d, L.in, key("k"), (int64_t)KH * dk, r0 + KQ, dk, a.DK));
  DEC_TRY(place_rows(d, L.in, key("v"), (int64_t)H * dv, r0 + 2 * KQ, dv, a.DV));
  DEC_TRY(place_rows(d, L.in, key("g"), (int64_t)H * dv, r0 + C, dv, a.DV));
  DEC_TRY(place_rows(d, L.in, key("b"), H, r0 + C + VW, H, H));
  DEC_TRY(place_rows(d, L.in, key("a"), H, r0 + C + VW + H, H, H));
  float *conv = nullptr, *taps = nullptr, *alog = nullptr, *na = nullptr, *v = nullptr;
  DEC_TRY(dev_alloc(d, (void **)&conv, sizeof(float) * (size_t)a.taps * C));
  struct { const char *key; int channels, ch0, hr, hrp; } parts[] = {
      {"q.conv", KH * dk, 0, dk, a.DK}, {"k.conv", KH * dk, KQ, dk, a.DK}, {"v.conv", H * dv, 2 * KQ, dv, a.DV}};
  for (auto &p : parts) {
    RawTensor *r = nullptr;
    DEC_TRY(raw_of(d, key(p.key), p.channels, a.taps, &r));
    DEC_TRY(to_f32(d, key(p.key), (int64_t)p.channels * a.taps, &taps));
    DEC_TRY(launch_place_taps(conv, taps, p.channels, a.taps, C, p.ch0, p.hr, p.hrp));
  }
  a.conv = conv;
  DEC_TRY(to_f32(d, key("A_log"), H, &alog));
  DEC_TRY(dev_alloc(d, (void **)&na, sizeof(float) * (size_t)H));
  DEC_TRY(launch_neg_exp(na, alog, H));
  a.neg_a = na;
  DEC_TRY(to_f32(d, key("dt_bias"), H, &v));
  a.dt_bias = v;
  DEC_TRY(vec_padded(d, key("norm"), dv, dv, a.DV, &v));
  a.norm = v;
  return 0;
}

static int load_latent(Decoder *d, int l, MixedBranch &br) {
  MixedLayer &L = d->mixed[l];
  const cthip_mixer_spec &sp = br.sp;
  const int H = sp.heads, dk = sp.dim, dv = sp.vdim, r = sp.kv_rank;
  auto key = [&](const char *k) { return mkey(l, br.prefix + k); };
  LatentArgs &a = br.latent;
  a.H = H, a.dk = dk, a.dv = dv, a.r = r, a.DK = pad16(dk), a.DV = pad16(dv), a.R = pad16(r);
  const int64_t r0 = br.row0;
  a.ldp = L.in->rows;
  a.eps = d->cfg.eps;
  a.scale = sp.scale;
  a.gated = sp.gate;
  int rc;
  RawTensor *uk = nullptr;
  DEC_TRY(place_rows(d, L.in, key("q"), (int64_t)H * dk, r0, dk, a.DK));
  DEC_TRY(place_rows(d, L.in, key("dkv"), r, r0 + (int64_t)H * a.DK, r, r));
  if (sp.gate) DEC_TRY(place_rows(d, L.in, key("g"), (int64_t)H * dv, r0 + (int64_t)H * a.DK + a.R, dv, a.DV));
  DEC_TRY(raw_of(d, key("uk"), (int64_t)H * dk, r, &uk));
  if (uk->type != L.in->type) return fail(CTHIP_E_BAD_ARG, "decoder: '%s' has ggml type %d, the layer's other weights %d", key("uk").c_str(), uk->type, L.in->type);
  DEC_TRY(wmat_empty(d, uk->type, (int64_t)H * a.R, a.DK, &br.absorb));
  DEC_TRY(launch_place_transposed(br.absorb->q, uk->dev, elem(br.absorb), H, dk, a.DK, r, a.R));
  DEC_TRY(wmat_empty(d, uk->type, (int64_t)H * (a.DK + a.DV), a.R, &br.kv_up));
  d->weight_bytes -= (int64_t)H * a.DK * a.R * elem(br.kv_up);  // (a decode step reads the key projection from `absorb` only)
  DEC_TRY(place_rows(d, br.kv_up, key("uk"), (int64_t)H * dk, 0, dk, a.DK, r));
  DEC_TRY(place_rows(d, br.kv_up, key("uv"), (int64_t)H * dv, (int64_t)H * a.DK, dv, a.DV, r));
  a.type = uk->type;
  a.absorb = br.absorb->q;
  a.up = (const char *)br.kv_up->q + (int64_t)H * a.DK * a.R * elem(br.kv_up);
  float *v = nullptr;
  DEC_TRY(vec_padded(d, key("dkv.norm"), r, r, a.R, &v));
  a.norm = v;
  if (sp.sink) {
    DEC_TRY(to_f32(d, key("sink"), H, &v));
    a.sink = v;
  }
  a.rows = d->cfg.max_seq;
  // key ranges of the decode attention: as many workgroups as there are compute units, at least a tile each
  int ranges = state().compute_units / ((H + 15) / 16);
  ranges = std::max(std::min({ranges, kLatentMaxRanges, (d->cfg.max_seq + 15) / 16}), 1);
  d->latent_work.ranges = d->latent_work.ranges ? std::min(d->latent_work.ranges, ranges) : ranges;
  return 0;
}

// the rotation of a window layer as a table over the session's positions; layers with the same one share it
typedef std::map<std::tuple<int, double, double, double, double, double>, float2 *> RopeTables;
static int rope_table(Decoder *d, const cthip_mixer_spec &sp, RopeTables &tables, float2 **out) {
  float2 *&t = tables[std::make_tuple(sp.rot_dims, sp.rot_base, sp.rot_factor, sp.rot_original, sp.rot_fast, sp.rot_slow)];
  if (!t) {
    const int dims = sp.rot_dims, half = dims / 2;
    std::vector<double> f(half);
    double lo = 0.0, hi = 0.0, mscale = 1.0;
    if (sp.rot_factor > 0.0) {
      // the pair (a real number) that turns `times` times over the original context
      auto pair = [&](double times) { return dims * log(sp.rot_original / (2.0 * M_PI * times)) / (2.0 * log(sp.rot_base)); };
      lo = std::max(floor(pair(sp.rot_fast)), 0.0);
      hi = std::min(ceil(pair(sp.rot_slow)), (double)dims - 1.0);
      mscale = 0.1 * log(sp.rot_factor) + 1.0;
    }
    for (int i = 0; i < half; i++) {
      f[i] = pow(sp.rot_base, -2.0 * i / dims);
      if (sp.rot_factor > 0.0) {
        const double ramp = std::min(std::max((i - lo) / std::max(hi - lo, 0.001), 0.0), 1.0);
        f[i] = f[i] / sp.rot_factor * ramp + f[i] * (1.0 - ramp);
      }
    }
    double *dev = nullptr;
    int rc;
    DEC_TRY(dev_alloc(d, (void **)&dev, sizeof(double) * (size_t)half));
    DEC_TRY(cthip_h2d(dev, f.data(), sizeof(double) * (size_t)half));
    DEC_TRY(dev_alloc(d, (void **)&t, sizeof(float2) * (size_t)d->cfg.max_seq * half));
    DEC_TRY(launch_rope_table(t, dev, d->cfg.max_seq, half, mscale));
  }
  *out = t;
  return 0;
}

static int load_window(Decoder *d, int l, MixedBranch &br, RopeTables &tables) {
  MixedLayer &L = d->mixed[l];
  const cthip_mixer_spec &sp = br.sp;
  const int H = sp.heads, G = sp.kv_heads, dk = sp.dim, dv = sp.vdim;
  auto key = [&](const char *k) { return mkey(l, br.prefix + k); };
  WindowArgs &a = br.window;
  a.H = H, a.G = G, a.dk = dk, a.dv = dv, a.DK = pad16(dk), a.DV = pad16(dv);
  a.window = sp.window;
  a.rows = std::min(sp.window, d->cfg.max_seq);
  a.ldp = L.in->rows;
  a.eps = d->cfg.eps;
  a.scale = sp.scale;
  a.out_scale = sp.out_scale;
  a.gated = sp.gate;
  const int64_t q0 = br.row0, k0 = q0 + (int64_t)H * a.DK, v0 = k0 + (int64_t)G * a.DK, g0 = v0 + (int64_t)G * a.DV;
  int rc;
  DEC_TRY(place_rows(d, L.in, key("q"), (int64_t)H * dk, q0, dk, a.DK));
  DEC_TRY(place_rows(d, L.in, key("k"), (int64_t)G * dk, k0, dk, a.DK));
  DEC_TRY(place_rows(d, L.in, key("v"), (int64_t)G * dv, v0, dv, a.DV));
  if (sp.gate) DEC_TRY(place_rows(d, L.in, key("g"), (int64_t)H * dv, g0, dv, a.DV));
  if (sp.bias) {
    if (!L.bias) DEC_TRY(dev_alloc(d, (void **)&L.bias, sizeof(float) * (size_t)L.in->rows));
    struct { const char *key; int64_t n, at; int hr, hrp; } parts[] = {
        {"q.b", (int64_t)H * dk, q0, dk, a.DK}, {"k.b", (int64_t)G * dk, k0, dk, a.DK}, {"v.b", (int64_t)G * dv, v0, dv, a.DV}};
    for (auto &p : parts) {
      float *b = nullptr;
      DEC_TRY(to_f32(d, key(p.key), p.n, &b));
      DEC_TRY(launch_place(L.bias, b, 4, p.n, 1, p.at, p.hr, p.hrp, 1, 1, 1));
    }
  }
  float *v = nullptr;
  if (sp.qk_norm) {
    DEC_TRY(vec_padded(d, key("q.norm"), (int64_t)H * dk, dk, a.DK, &v));
    a.qnorm = v;
    DEC_TRY(vec_padded(d, key("k.norm"), (int64_t)G * dk, dk, a.DK, &v));
    a.knorm = v;
  }
  if (sp.sink == CTHIP_SINK_TENSOR) {
    DEC_TRY(to_f32(d, key("sink"), H, &v));
    a.sink = v;
  } else if (sp.sink == CTHIP_SINK_ZERO) {
    DEC_TRY(dev_alloc(d, (void **)&v, sizeof(float) * (size_t)H));  // (zero-filled)
    a.sink = v;
  }
  if (sp.rot_dims) {
    float2 *t = nullptr;
    DEC_TRY(rope_table(d, sp, tables, &t));
    a.rope = t;
    a.half = sp.rot_dims / 2;
  }
  return 0;
}

static int load_lightning(Decoder *d, int l, MixedBranch &br) {
  MixedLayer &L = d->mixed[l];
  const cthip_mixer_spec &sp = br.sp;
  const int H = sp.heads, dk = sp.dim, dv = sp.vdim;
  auto key = [&](const char *k) { return mkey(l, br.prefix + k); };
  LightningArgs &a = br.lightning;
  a.H = H, a.dk = dk, a.dv = dv, a.DK = pad16(dk), a.DV = pad16(dv);
  a.ldp = L.in->rows;
  a.eps = d->cfg.eps;
  a.out_scale = sp.out_scale;
  const int64_t q0 = br.row0, k0 = q0 + (int64_t)H * a.DK, v0 = k0 + (int64_t)H * a.DK, g0 = v0 + (int64_t)H * a.DV;
  int rc;
  DEC_TRY(place_rows(d, L.in, key("q"), (int64_t)H * dk, q0, dk, a.DK));
  DEC_TRY(place_rows(d, L.in, key("k"), (int64_t)H * dk, k0, dk, a.DK));
  DEC_TRY(place_rows(d, L.in, key("v"), (int64_t)H * dv, v0, dv, a.DV));
  DEC_TRY(place_rows(d, L.in, key("g"), (int64_t)H * dv, g0, dv, a.DV));
  float *v = nullptr;
  DEC_TRY(vec_padded(d, key("norm"), (int64_t)H * dv, dv, a.DV, &v));
  a.norm = v;
  std::vector<float> dec(3 * (size_t)H);
  for (int h = 0; h < H; h++) {
    const double g = br.decay[h];
    dec[h] = (float)(g - 1.0);
    dec[H + h] = (float)(g > 0.0 ? log2(g) : -1e4);  // (2^(-1e4 n) is zero from n = 1 on, and one at n = 0)
    dec[2 * H + h] = (float)g;
  }
  DEC_TRY(dev_alloc(d, (void **)&v, sizeof(float) * dec.size()));
  DEC_TRY(cthip_h2d(v, dec.data(), sizeof(float) * dec.size()));
  a.decay = v;
  return 0;
}

// what a layer run keeps of the sequence
static int keep_alloc(Decoder *d, const MixedBranch &br, float *keep[2]) {
  size_t n0 = 0, n1 = 0;
  switch (br.sp.mixer) {
    case CTHIP_MIXER_DELTA:
      n0 = (size_t)br.delta.taps * br.delta.C;
      n1 = (size_t)br.delta.H * br.delta.DV * br.delta.DK;
      break;
    case CTHIP_MIXER_LATENT: n0 = (size_t)br.latent.rows * br.latent.R; break;
    case CTHIP_MIXER_WINDOW:
      n0 = (size_t)br.window.rows * br.window.G * br.window.DK;
      n1 = (size_t)br.window.rows * br.window.G * br.window.DV;
      break;
    default: n0 = (size_t)br.lightning.H * br.lightning.DV * br.lightning.DK;
  }
  int rc;
  DEC_TRY(dev_alloc(d, (void **)&keep[0], sizeof(float) * n0));
  if (n1) DEC_TRY(dev_alloc(d, (void **)&keep[1], sizeof(float) * n1));
  return 0;
}
// a branch's arguments for one run over the projection rows p (the layer's)
static DeltaArgs delta_of(const MixedBranch &br, float *const *keep, const float *p) {
  DeltaArgs a = br.delta;
  a.p = p + br.row0, a.ring = keep[0], a.S = keep[1];
  return a;
}
static LatentArgs latent_of(const MixedBranch &br, float *const *keep, const float *p) {
  LatentArgs a = br.latent;
  a.p = p + br.row0, a.cache = keep[0];
  return a;
}
static WindowArgs window_of(const MixedBranch &br, float *const *keep, const float *p) {
  WindowArgs a = br.window;
  a.p = p + br.row0, a.K = keep[0], a.V = keep[1];
  return a;
}
static LightningArgs lightning_of(const MixedBranch &br, float *const *keep, const float *p) {
  LightningArgs a = br.lightning;
  a.p = p + br.row0, a.S = keep[0];
  return a;
}

int mixed_load(Decoder *d) {
  const cthip_decoder_config &c = d->cfg;
  const cthip_mixed_config &mc = d->mcfg;
  const int D = c.dim, V = c.vocab;
  const bool ln = mc.norm == CTHIP_PRO_LAYERNORM;
  int rc;
  auto norm = [&](const std::string &key, float **out) {
    const int r = to_f32(d, key, D, out);
    return r || !mc.norm_plus_one ? r : launch_add_one(*out, D);
  };
  DEC_TRY(to_f32(d, "embed", (int64_t)V * D, &d->wte));
  if (mc.position_base > 0.0f) {
    DEC_TRY(dev_alloc(d, (void **)&d->wpe, sizeof(float) * (size_t)c.max_seq * D));
    DEC_TRY(launch_sinusoid_table(d->wpe, c.max_seq, D, mc.position_base));
  }
  DEC_TRY(norm("final.norm", &d->lnf_g));
  DEC_TRY(to_wmat(d, {mc.tied_head ? "embed" : "head"}, V, D, &d->lm_head));
  float *none = nullptr;
  if (ln) DEC_TRY(make_fold(d, d->lm_head, d->lnf_g, nullptr, nullptr, &d->lm_s, &none));
  int64_t most_p = 0, most_o = 0, most_h = 0, most_qa = 0, most_part = 0, most_win = 0, most_raw = 0;
  int tickets = 0;
  RopeTables tables;
  for (int l = 0; l < c.n_layers; l++) {
    MixedLayer &L = d->mixed[l];
    const cthip_layer_spec &sp = L.sp;
    const int64_t before = d->weight_bytes + d->vector_bytes;
    DEC_TRY(norm(mkey(l, "norm1"), &L.norm1));
    int64_t rows = 0, cols = 0;
    for (MixedBranch &br : L.branches) {
      br.row0 = rows, br.col0 = cols;
      rows += branch_rows(br.sp);
      cols += (int64_t)br.sp.heads * pad16(br.sp.vdim);
    }
    DEC_TRY(in_matrix(d, l, rows));
    for (MixedBranch &br : L.branches) {
      const int64_t H = br.sp.heads;
      if (br.sp.mixer == CTHIP_MIXER_DELTA) {
        DEC_TRY(load_delta(d, l, br));
      } else if (br.sp.mixer == CTHIP_MIXER_LATENT) {
        DEC_TRY(load_latent(d, l, br));
        most_qa = std::max(most_qa, H * br.latent.R);
        most_part = std::max(most_part, (int64_t)latent_part_floats((int)H, br.latent.R, kLatentMaxRanges));
      } else if (br.sp.mixer == CTHIP_MIXER_WINDOW) {
        DEC_TRY(load_window(d, l, br, tables));
        most_win = std::max(most_win, (int64_t)window_part_floats(br.window));
        tickets = std::max(tickets, window_tickets(br.window));
      } else {
        DEC_TRY(load_lightning(d, l, br));
        most_raw = std::max(most_raw, (int64_t)lightning_raw_floats(br.lightning));
      }
    }
    if (ln) {
      if (L.bias) return fail(CTHIP_E_UNSUPPORTED, "decoder: projections with biases behind a LayerNorm");
      DEC_TRY(make_fold(d, L.in, L.norm1, nullptr, nullptr, &L.in_s, &none));
    }
    for (const MixedBranch &br : L.branches) {
      const int64_t H = br.sp.heads, dv = br.sp.vdim, DV = pad16(br.sp.vdim);
      const std::string key = mkey(l, br.prefix + "o");
      RawTensor *o = nullptr;
      DEC_TRY(raw_of(d, key, D, H * dv, &o));
      if (!L.out) DEC_TRY(wmat_empty(d, o->type, D, cols, &L.out));
      if (o->type != L.out->type) return fail(CTHIP_E_BAD_ARG, "decoder: tensor '%s' has ggml type %d, its neighbours %d", key.c_str(), o->type, L.out->type);
      DEC_TRY(launch_place((char *)L.out->q + br.col0 * elem(L.out), o->dev, elem(L.out), D, H * dv, 0, D, D, dv, DV, cols));
    }
    if (sp.layer_scale) DEC_TRY(to_f32(d, mkey(l, "ls1"), D, &L.ls1));
    if (sp.ffn) {
      DEC_TRY(norm(mkey(l, "norm2"), &L.norm2));
      RawTensor *g = nullptr;
      DEC_TRY(raw_of(d, mkey(l, "mlp.gate"), sp.ffn, D, &g));
      L.fc_pairs = gemv_pair_swiglu_ok(g->type, 2 * (int64_t)sp.ffn, D, ln);
      DEC_TRY(to_wmat(d, {mkey(l, "mlp.gate"), mkey(l, "mlp.up")}, 2 * (int64_t)sp.ffn, D, &L.gate_up, L.fc_pairs));
      DEC_TRY(to_wmat(d, {mkey(l, "mlp.down")}, D, sp.ffn, &L.down));
      if (ln) DEC_TRY(make_fold(d, L.gate_up, L.norm2, nullptr, nullptr, &L.fc_s, &none));
      if (sp.layer_scale) DEC_TRY(to_f32(d, mkey(l, "ls2"), D, &L.ls2));
    }
    L.nbytes = d->weight_bytes + d->vector_bytes - before;
    most_p = std::max(most_p, rows);
    most_o = std::max(most_o, cols);
    most_h = std::max(most_h, 2 * (int64_t)sp.ffn);
  }
  for (MixedRun &r : d->runs)
    for (size_t b = 0; b < d->mixed[r.layer].branches.size(); b++) DEC_TRY(keep_alloc(d, d->mixed[r.layer].branches[b], r.keep[b]));
  DEC_TRY(dev_alloc(d, (void **)&d->q, sizeof(float) * (size_t)most_p));
  DEC_TRY(dev_alloc(d, (void **)&d->att, sizeof(float) * (size_t)most_o));
  if (most_h) DEC_TRY(dev_alloc(d, (void **)&d->h, sizeof(float) * (size_t)most_h));
  if (most_qa) {
    DEC_TRY(dev_alloc(d, (void **)&d->latent_work.qa, sizeof(float) * (size_t)most_qa));
    DEC_TRY(dev_alloc(d, (void **)&d->latent_work.part, sizeof(float) * (size_t)most_part));
  }
  if (most_win) DEC_TRY(dev_alloc(d, (void **)&d->parallel_work.part, sizeof(float) * (size_t)most_win));
  if (most_raw) DEC_TRY(dev_alloc(d, (void **)&d->parallel_work.raw, sizeof(float) * (size_t)most_raw));
  if (most_win || most_raw) DEC_TRY(dev_alloc(d, (void **)&d->parallel_work.count, sizeof(int) * (size_t)(1 + tickets)));  // (zero-filled)
  return 0;
}

void mixed_release(Decoder *d) {
  for (MixedLayer &L : d->mixed) {
    for (WMat *w : {L.in, L.out, L.gate_up, L.down}) cthip_wmat_destroy(w);
    for (MixedBranch &br : L.branches)
      for (WMat *w : {br.absorb, br.kv_up}) cthip_wmat_destroy(w);
  }
}

int mixed_launches(const Decoder *d) {
  int most = 0;
  for (const MixedLayer &L : d->mixed) most = std::max(most, (L.branches[0].sp.mixer == CTHIP_MIXER_LATENT ? 5 : 3) + (L.sp.ffn ? 2 : 0));
  return most;
}

int64_t mixed_state_bytes(const Decoder *d, int t) {
  int64_t n = 0;
  std::vector<int> seen(d->mixed.size(), 0);
  for (const MixedRun &r : d->runs) {
    const MixedLayer &L = d->mixed[r.layer];
    if (seen[r.layer]++) n += L.nbytes;  // (the session's total counts every weight once)
    if (r.add_embedding) n += 4ll * d->cfg.dim;
    for (const MixedBranch &br : L.branches) {
      if (br.sp.mixer == CTHIP_MIXER_DELTA) n += 4 * (2ll * br.delta.H * br.delta.DV * br.delta.DK + (int64_t)br.delta.taps * br.delta.C);
      else if (br.sp.mixer == CTHIP_MIXER_LATENT) n += 4 * (int64_t)(t + 1) * br.latent.R;
      else if (br.sp.mixer == CTHIP_MIXER_WINDOW) n += 4 * (int64_t)std::min(t + 1, br.window.rows) * br.window.G * (br.window.DK + br.window.DV);
      else n += 4 * 2ll * br.lightning.H * br.lightning.DV * br.lightning.DK;
    }
  }
  return n;
}

int mixed_peek(Decoder *d, const char *what, void **ptr, int64_t *n_floats) {
  int r = -1;
  auto run_of = [&](const char *form) { return sscanf(what, form, &r) == 1 && r >= 0 && r < (int)d->runs.size(); };
  const bool latent = run_of("latent.%d"), st = !latent && run_of("state.%d"), keys = !latent && !st && run_of("keys.%d"),
             values = !latent && !st && !keys && run_of("values.%d");
  if (!latent && !st && !keys && !values) return 1;
  const MixedLayer &L = d->mixed[d->runs[r].layer];
  for (size_t b = 0; b < L.branches.size(); b++) {
    const MixedBranch &br = L.branches[b];
    float *const *keep = d->runs[r].keep[b];
    int64_t n = 0;
    float *p = nullptr;
    if (latent && br.sp.mixer == CTHIP_MIXER_LATENT) p = keep[0], n = (int64_t)d->cfg.max_seq * br.latent.R;
    else if (st && br.sp.mixer == CTHIP_MIXER_DELTA) p = keep[1], n = (int64_t)br.delta.H * br.delta.DV * br.delta.DK;
    else if (st && br.sp.mixer == CTHIP_MIXER_LIGHTNING) p = keep[0], n = (int64_t)br.lightning.H * br.lightning.DV * br.lightning.DK;
    else if (keys && br.sp.mixer == CTHIP_MIXER_WINDOW) p = keep[0], n = (int64_t)br.window.rows * br.window.G * br.window.DK;
    else if (values && br.sp.mixer == CTHIP_MIXER_WINDOW) p = keep[1], n = (int64_t)br.window.rows * br.window.G * br.window.DV;
    if (!p) continue;
    *ptr = p;
    if (n_floats) *n_floats = n;
    return 0;
  }
  return 1;
}

int mixed_queue_layers(Decoder *d) {
  const int D = d->cfg.dim, pro = d->mcfg.norm;
  const int *pos = d->tokpos + 1;
  int rc;
  auto normed = [&](const WMat *w, const float *g, const float *fold, const float *bias, float *y, const Glu *pairs) {
    GemvArgs a = {};
    a.x = d->x;
    a.pro = pro;
    a.norm_g = g;
    a.eps = d->cfg.eps;
    a.fold_s = fold;
    a.bias = bias;
    if (pairs) a.pair_swiglu = 1, a.glu = *pairs;
    a.y = y;
    a.x_stride = D;
    a.y_stride = pairs ? w->rows / 2 : w->rows;
    return launch_gemv(w, a, 1);
  };
  auto residual = [&](const WMat *w, const float *x, const float *scale, const Glu *gate) {
    GemvArgs a = {};
    a.x = x;
    if (gate) a.pro = CTHIP_PRO_SWIGLU, a.glu = *gate;
    a.residual = d->x;
    a.row_scale = scale;
    a.y = d->x;
    a.x_stride = gate ? 2 * w->cols : w->cols;
    a.y_stride = D;
    return launch_gemv(w, a, 1);
  };
  for (MixedRun &r : d->runs) {
    MixedLayer &L = d->mixed[r.layer];
    if (r.add_embedding) DEC_TRY(launch_add_embedding(d->x, d->wte, d->wpe, d->tokpos, pos, 1, d->cfg.vocab, D, d->cfg.max_seq));
    DEC_TRY(normed(L.in, L.norm1, L.in_s, L.bias, d->q, nullptr));
    const int kind = L.branches[0].sp.mixer;
    if (kind == CTHIP_MIXER_DELTA) {
      DEC_TRY(launch_delta_step(delta_of(L.branches[0], r.keep[0], d->q), d->att, d->tokpos, d->ctrl));
    } else if (kind == CTHIP_MIXER_LATENT) {
      DEC_TRY(launch_latent_step(latent_of(L.branches[0], r.keep[0], d->q), d->latent_work, d->att, pos));
    } else {
      // a window and a lightning branch go into one launch; two of one kind are a launch each
      WindowArgs w;
      LightningArgs n;
      float *wout = nullptr, *nout = nullptr;
      for (size_t b = 0; b < L.branches.size(); b++) {
        const MixedBranch &br = L.branches[b];
        const bool win = br.sp.mixer == CTHIP_MIXER_WINDOW;
        if (win ? wout : nout) {
          DEC_TRY(launch_parallel_step(wout ? &w : nullptr, wout, nout ? &n : nullptr, nout, d->parallel_work, d->tokpos, d->ctrl));
          wout = nout = nullptr;
        }
        if (win) w = window_of(br, r.keep[b], d->q), wout = d->att + br.col0;
        else n = lightning_of(br, r.keep[b], d->q), nout = d->att + br.col0;
      }
      DEC_TRY(launch_parallel_step(wout ? &w : nullptr, wout, nout ? &n : nullptr, nout, d->parallel_work, d->tokpos, d->ctrl));
    }
    DEC_TRY(residual(L.out, d->att, L.ls1, nullptr));
    if (L.sp.ffn) {
      DEC_TRY(normed(L.gate_up, L.norm2, L.fc_s, nullptr, d->h, L.fc_pairs ? &L.glu : nullptr));
      DEC_TRY(residual(L.down, d->h, L.ls2, L.fc_pairs ? nullptr : &L.glu));
    }
  }
  return 0;
}

int mixed_prefill(Decoder *d, float *X, float *XN, const int *ids, int s, int n) {
  const cthip_decoder_config &c = d->cfg;
  const int D = c.dim;
  const bool rms = d->mcfg.norm == CTHIP_PRO_RMSNORM;
  const int prec = d->mcfg.precision >= 0 ? d->mcfg.precision : state().gemm_precision;
  size_t most_p = 0, most_o = 0, most_h = 0, most_g = 0, most_w = 0;
  for (const MixedLayer &L : d->mixed) {
    most_p = std::max(most_p, (size_t)s * L.in->rows);
    most_o = std::max(most_o, (size_t)s * L.out->cols);
    for (const MixedBranch &br : L.branches) {
      size_t w = 0;
      switch (br.sp.mixer) {
        case CTHIP_MIXER_DELTA: w = delta_scratch_floats(br.delta, s); break;
        case CTHIP_MIXER_LATENT: w = (size_t)(n + s) * br.kv_up->rows; break;
        case CTHIP_MIXER_WINDOW: w = (size_t)(window_prev(br.window, n) + s) * br.window.G * (br.window.DK + br.window.DV); break;
        default: w = lightning_scratch_floats(br.lightning, s);
      }
      most_w = std::max(most_w, w);
    }
    if (L.sp.ffn) most_h = std::max(most_h, (size_t)s * 2 * L.sp.ffn), most_g = std::max(most_g, (size_t)s * L.sp.ffn);
  }
  float *P = nullptr, *O = nullptr, *Hb = nullptr, *G = nullptr, *W = nullptr;
  int rc = 0;
  auto norm = [&](const float *g) { return rms ? cthip_rmsnorm(XN, X, g, c.eps, s, D) : cthip_layernorm(XN, X, g, nullptr, c.eps, s, D); };
  auto latent_rows = [&](const MixedBranch &br, float *const *keep, int64_t ldo) -> int {
    const LatentArgs a = latent_of(br, keep, P);
    int rc;
    DEC_TRY(launch_latent_append(a, s, n));
    // keys and values of every visible row
    DEC_TRY(launch_linear_gemm(W, br.kv_up, a.cache, n + s, nullptr, nullptr, CTHIP_ACT_NONE, prec));
    AttnRowsArgs r = {};
    r.out = O + br.col0;
    r.q = a.p;
    r.k = W;
    r.v = W + (size_t)a.H * a.DK;
    r.S = s;
    r.start_pos = n;
    r.H = r.Hkv = a.H;
    r.ldq = r.ldg = (int)a.ldp;
    r.ldk = r.ldv = (int)br.kv_up->rows;
    r.dk = a.DK;
    r.dv = a.DV;
    r.scale = a.scale;
    r.sink = a.sink;
    r.gate = a.gated ? a.p + (size_t)a.H * a.DK + a.R : nullptr;
    r.ldo = (int)ldo;
    return launch_attn_rows(r, prec == GEMM_FP32);
  };
  auto window_rows = [&](const MixedBranch &br, float *const *keep, int64_t ldo) -> int {
    const WindowArgs a = window_of(br, keep, P);
    const int prev = window_prev(a, n);
    float *kb = W, *vb = W + (size_t)(prev + s) * a.G * a.DK;
    int rc;
    DEC_TRY(launch_window_prepare(a, P + br.row0, kb, vb, s, n));
    AttnRowsArgs r = {};
    r.out = O + br.col0;
    r.q = a.p;
    r.k = kb;
    r.v = vb;
    r.S = s;
    r.start_pos = prev;
    r.H = a.H;
    r.Hkv = a.G;
    r.ldq = r.ldg = (int)a.ldp;
    r.ldk = a.G * a.DK;
    r.ldv = a.G * a.DV;
    r.dk = a.DK;
    r.dv = a.DV;
    r.scale = a.scale;
    r.sink = a.sink;
    r.window = a.window;
    r.out_scale = a.out_scale;
    r.gate = a.gated ? a.p + (size_t)a.H * a.DK + (size_t)a.G * (a.DK + a.DV) : nullptr;
    r.ldo = (int)ldo;
    DEC_TRY(launch_attn_rows(r, prec == GEMM_FP32));
    return launch_window_keep(a, kb, vb, s, n);
  };
  auto run = [&]() -> int {
    int rc;
    DEC_TRY(alloc_scratch((void **)&P, sizeof(float) * most_p));
    DEC_TRY(alloc_scratch((void **)&O, sizeof(float) * most_o));
    DEC_TRY(alloc_scratch((void **)&W, sizeof(float) * most_w));
    if (most_h) {
      DEC_TRY(alloc_scratch((void **)&Hb, sizeof(float) * most_h));
      DEC_TRY(alloc_scratch((void **)&G, sizeof(float) * most_g));
    }
    DEC_TRY(norm(d->mixed[d->runs[0].layer].norm1));
    for (size_t k = 0; k < d->runs.size(); k++) {
      const MixedRun &r = d->runs[k];
      MixedLayer &L = d->mixed[r.layer];
      if (r.add_embedding) {
        DEC_TRY(launch_add_embedding(X, d->wte, d->wpe, ids, d->tokpos + 1, s, c.vocab, D, c.max_seq));
        DEC_TRY(norm(L.norm1));
      }
      DEC_TRY(launch_linear_gemm(P, L.in, XN, s, L.bias, nullptr, CTHIP_ACT_NONE, prec));
      for (size_t b = 0; b < L.branches.size(); b++) {
        const MixedBranch &br = L.branches[b];
        switch (br.sp.mixer) {
          case CTHIP_MIXER_DELTA: rc = launch_delta_rows(delta_of(br, r.keep[b], P), O, s, n, W); break;
          case CTHIP_MIXER_LATENT: rc = latent_rows(br, r.keep[b], L.out->cols); break;
          case CTHIP_MIXER_WINDOW: rc = window_rows(br, r.keep[b], L.out->cols); break;
          default: rc = launch_lightning_rows(lightning_of(br, r.keep[b], P), O + br.col0, L.out->cols, s, n, W);
        }
        if (rc) return rc;
      }
      // the norm in front of what comes next; the embedding goes in between where the next run starts a pass
      const bool more = k + 1 < d->runs.size() && !d->runs[k + 1].add_embedding;
      const float *next = more ? d->mixed[d->runs[k + 1].layer].norm1 : nullptr;
      DEC_TRY(linear_residual_norm(XN, X, L.out, O, s, D, nullptr, L.sp.ffn ? L.norm2 : next, nullptr, c.eps, rms, prec, L.ls1));
      if (L.sp.ffn) {
        const int F = L.sp.ffn;
        if (L.fc_pairs && (2 * F) % 4 == 0) {
          DEC_TRY(launch_linear_gemm(G, L.gate_up, XN, s, nullptr, nullptr, kActSwigluPairs, prec, nullptr, nullptr, nullptr, L.glu));
        } else {
          DEC_TRY(launch_linear_gemm(Hb, L.gate_up, XN, s, nullptr, nullptr, CTHIP_ACT_NONE, prec));
          if (L.fc_pairs) DEC_TRY(launch_swiglu_pairs(G, Hb, (int64_t)s * F, L.glu));
          else DEC_TRY(launch_prologue(G, Hb, F, CTHIP_PRO_SWIGLU, nullptr, nullptr, 0.0f, 2 * (int64_t)F, s, L.glu));
        }
        DEC_TRY(linear_residual_norm(XN, X, L.down, G, s, D, nullptr, next, nullptr, c.eps, rms, prec, L.ls2));
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
