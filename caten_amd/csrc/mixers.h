// The token mixers of decoders whose layers are listed one by one: the gated delta rule (delta.hip) and attention over
// a cached latent vector (latent.hip).  Head sizes are padded to multiples of 16 in memory (zero rows and columns of
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
// dst[i] = src[rows[i]] for rows of n floats
int launch_gather_rows(float *dst, const float *src, const int *rows, int nrows, int n);

}  // namespace cthip
