// The token mixers of decoders whose layers are listed one by one: the gated delta rule (delta.hip), attention over
// a cached latent vector (latent.hip), attention over a sliding window and lightning attention (window.hip, lightning.hip;
// parallel.hip runs a decode step of the two side by side).  Head sizes are padded to multiples of 16 in memory (zero rows and columns of
// the weights), so every row of a head is whole 16-byte pieces; the true sizes matter only where a mean is taken.
#pragma once
#include "common.h"

namespace cthip {

constexpr int pad16(int n) { return (n + 15) & ~15; }

// ---- gated delta rule ----
// A projection row holds [q: KH x DK | k: KH x DK | v: H x DV | g: H x DV | b: H | a: H]; its first C = 2 KH DK + H DV
// entries pass the short convolution and are what the history keeps of a token.
struct DeltaArgs {
  const float *p;   // projection rows, ldp floats apart
  int64_t ldp;
  int H, KH, DK, DV, dk, dv, taps, C;
  const float *conv;      // [taps][C]: row j meets the token j steps back
  float *ring;            // [taps][C]: the raw row of position i at slot i mod taps
  float *S;               // [H][DV][DK], fp32
  const float *neg_a;     // [H]: -exp(A_log)
  const float *dt_bias;   // [H]
  const float *norm;      // [DV], zeros in the padding
  float eps;
};
// one token at position tokpos[1]: convolutions, state update, read-out, norm and gate -> out (H x DV); the state and the
// history stay as they are once ctrl[1] is set (the sequence has ended)
int launch_delta_step(const DeltaArgs &a, float *out, const int *tokpos, const int *ctrl);
// s tokens at positions n .. n + s - 1 -> out (s, H x DV); scratch: delta_scratch_floats() floats
size_t delta_scratch_floats(const DeltaArgs &a, int s);
int launch_delta_rows(const DeltaArgs &a, float *out, int s, int n, float *scratch);

// ---- attention over a cached latent ----
// A projection row holds [q: H x DK | latent: R | g: H x DV, where the output is gated]; the cache keeps the normalised latent, R floats a row.
struct LatentArgs {
  const float *p;
  int64_t ldp;
  int H, DK, DV, R, r, dk, dv;
  float eps, scale;
  const float *norm;   // [R], zeros in the padding
  int gated;           // the output is multiplied by sigmoid(g)
  const float *sink;   // [H] logits of the extra softmax term (no key, no value); null = none
  float *cache;        // [rows][R]
  int rows;
  int type;            // weight type of absorb / up
  const void *absorb;  // [H][R][DK]: the key projection, transposed per head
  const void *up;      // [H][DV][R]: the value projection
};
constexpr int kLatentMaxRanges = 128;
struct LatentWork {
  float *qa;    // [H][R]: queries carried into the latent space
  float *part;  // [ranges][H]: unnormalised sums, maximum and denominator of every key range (latent_part_floats)
  int ranges;
};
size_t latent_part_floats(int H, int R, int ranges);
// one token at position *pos: appends its latent, attends over rows 0 .. *pos, gates -> out (H x DV); three launches
int launch_latent_step(const LatentArgs &a, const LatentWork &w, float *out, const int *pos);
// appends the latents of s tokens at rows n ..
int launch_latent_append(const LatentArgs &a, int s, int n);

// ---- attention over a sliding window ----
// A projection row holds [q: H x DK | k: G x DK | v: G x DV | g: H x DV, where the output is gated].  Keys and values of
// the last `rows` positions are kept in rings: position i in row i mod rows.
struct WindowArgs {
  const float *p;
  int64_t ldp;
  int H, G, DK, DV, dk, dv;
  int window, rows;        // rows = min(window, longest sequence)
  float eps, scale, out_scale;
  const float *qnorm, *knorm;  // [H x DK], [G x DK], zeros in the padding; null = no norm
  const float2 *rope;      // [position][half]: cosine and sine; null = no rotation
  int half;                // entries i and i + half of a head are a pair, i < half
  const float *sink;       // [H] logits of the extra softmax term; null = none
  int gated;
  float *K, *V;            // [rows][G x DK], [rows][G x DV]
};
// queries and keys of s rows normalised and rotated, queries in place; keys and values of the visible earlier rows and of
// these -> kbuf (prev + s, G x DK), vbuf (prev + s, G x DV), prev = window_prev(a, n)
int window_prev(const WindowArgs &a, int n);
int launch_window_prepare(const WindowArgs &a, float *p, float *kbuf, float *vbuf, int s, int n);
// the last rows of kbuf / vbuf into the rings
int launch_window_keep(const WindowArgs &a, const float *kbuf, const float *vbuf, int s, int n);

// ---- lightning attention ----
// A projection row holds [q: H x DK | k: H x DK | v: H x DV | g: H x DV].
struct LightningArgs {
  const float *p;
  int64_t ldp;
  int H, DK, DV, dk, dv;
  const float *decay;      // [3][H]: the decay less 1, its logarithm to base 2, the decay itself
  const float *norm;       // [H x DV], zeros in the padding
  float eps, out_scale;
  float *S;                // [H][DV][DK], fp32
};
// s tokens at positions n .. n + s - 1 -> out rows ldo floats apart; scratch: lightning_scratch_floats() floats
size_t lightning_scratch_floats(const LightningArgs &a, int s);
int launch_lightning_rows(const LightningArgs &a, float *out, int64_t ldo, int s, int n, float *scratch);

// ---- a decode step of either, or of both side by side in one launch ----
struct ParallelWork {
  float *part;   // window: every key range's unnormalised sums, maximum and denominator
  int *count;    // tickets: one for the lightning heads, then window_tickets() of them; zeroed (each launch leaves them zeroed again)
  float *raw;    // lightning: H x DV outputs before the norm
};
constexpr int kWindowMaxRanges = 32;
int window_tickets(const WindowArgs &a);
size_t window_part_floats(const WindowArgs &a);
size_t lightning_raw_floats(const LightningArgs &a);
// w -> wout (H x DV), l -> lout (H x DV); either may be null.  The token at position tokpos[1]; once ctrl[1] is set (the
// sequence has ended) the recurrent state stays as it is
int launch_parallel_step(const WindowArgs *w, float *wout, const LightningArgs *l, float *lout, const ParallelWork &work,
                         const int *tokpos, const int *ctrl);

// ---- attention of prompt rows with key and value heads of different sizes (attn_rows_*.hip) ----
struct AttnRowsArgs {
  float *out;             // (S, H x dv), ldo floats apart
  const float *q, *k, *v; // rows ldq / ldk / ldv floats apart, heads dk / dk / dv floats apart
  int S, start_pos, H, Hkv;
  int ldq, ldk, ldv, ldo, ldg;
  int dk, dv;             // multiples of 4, at most 256
  float scale;
  const float *sink;      // [H] or null
  const float *gate;      // (S, H x dv) rows ldg apart or null: the output is multiplied by its sigmoid
  int window;             // > 0: a row sees its last `window` keys only, itself included
  float out_scale = 1.0f; // a factor of the output
};
int launch_attn_rows(const AttnRowsArgs &a, bool fp32_operands);
int launch_attn_rows_f32(const AttnRowsArgs &a);
int launch_attn_rows_bf(const AttnRowsArgs &a);

// ---- small pieces ----
// dst[(r0 + (i / hr) * hrp + i % hr) * ld + (j / hc) * hcp + j % hc] = src[i][j] for a (rows, cols) matrix of `es`-byte
// elements: rows in heads of hr placed hrp apart, columns in heads of hc placed hcp apart
int launch_place(void *dst, const void *src, int es, int64_t rows, int64_t cols, int64_t r0, int64_t hr, int64_t hrp, int64_t hc,
                 int64_t hcp, int64_t ld);
// dst[h][c][r] = src[h * hr + r][c] (r < hr padded to hrp, c < cols padded to colsp): every head's block transposed
int launch_place_transposed(void *dst, const void *src, int es, int64_t heads, int64_t hr, int64_t hrp, int64_t cols, int64_t colsp);
// table[p][2i] = sin(p base^(-2i / dim)), [2i + 1] = cos of the same
int launch_sinusoid_table(float *table, int rows, int dim, double base);
// dst[t][ch0 + i] = w[i][taps - 1 - t] of an fp32 (channels, taps) tensor, channels in heads of hr placed hrp apart
int launch_place_taps(float *dst, const float *w, int channels, int taps, int C, int ch0, int hr, int hrp);
int launch_neg_exp(float *y, const float *x, int n);
int launch_softcap(float *y, int64_t n, float cap);
// x[i] += 1 for a norm weight that is stored around zero
int launch_add_one(float *x, int n);
// table[p][i] = (cos, sin)(p freqs[i]) * mscale, computed in double precision
int launch_rope_table(float2 *table, const double *freqs, int rows, int half, double mscale);
// x[t] += wte[ids[t]] (+ wpe[pos[0] + t]) for `ntok` rows of n floats (an id outside the vocabulary selects no row)
int launch_add_embedding(float *x, const float *wte, const float *wpe, const int *ids, const int *pos, int ntok, int vocab, int n, int max_pos);
// dst[i] = src[rows[i]] for rows of n floats
int launch_gather_rows(float *dst, const float *src, const int *rows, int nrows, int n);

}  // namespace cthip
