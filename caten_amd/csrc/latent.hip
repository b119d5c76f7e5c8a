// Attention over a cached latent: a token leaves one normalised vector c of R floats in the cache, and every head's keys
// and values are linear maps of it (k = W_uk c, v = W_uv c).  The softmax may have a sink: one logit per head that takes
// part in the denominator and has no value.  The concatenated heads are multiplied by the sigmoid of a gate.
//
// Decode never forms keys or values: q . (W_uk c) = (W_uk^T q) . c, and sum_j p_j (W_uv c_j) = W_uv (sum_j p_j c_j).
//   k_latent_absorb   qa_h = W_uk_h^T q_h for every head; one more workgroup normalises the new latent into the cache
//   k_latent_attend   all heads against a range of the cached rows: every cached row is read for 16 heads at once, on
//                     v_mfma_f32_16x16x4_f32 (fp32 products); leaves unnormalised sums, maxima and denominators
//   k_latent_up       merges the ranges and the sink, multiplies by W_uv, applies the gate
// Prompts expand the keys and values of all visible rows with one GEMM and attend as prompt rows do (attn_rows.h).
#include "common.h"
#include "mixers.h"

namespace cthip {

typedef float v4f_t __attribute__((ext_vector_type(4)));

// one lane's share (16-byte pieces l, l + 16, ...) of a row times a vector; TYPE: fp32, fp16 or bf16 weights
template <int TYPE>
__device__ __forceinline__ float row_dot16(const void *__restrict__ w, int64_t row, const float *__restrict__ x, int n, int l) {
  float acc = 0.0f;
  if (TYPE == CTHIP_F32) {
    const float4 *wr = (const float4 *)((const float *)w + row * n);
    const float4 *x4 = (const float4 *)x;
#pragma unroll 4
    for (int i = l; i < (n >> 2); i += 16) {
      const float4 a = wr[i], b = x4[i];
      acc = fmaf(a.x, b.x, fmaf(a.y, b.y, fmaf(a.z, b.z, fmaf(a.w, b.w, acc))));
    }
  } else {
    const uint4 *wr = (const uint4 *)((const unsigned short *)w + row * n);
    const float4 *x4 = (const float4 *)x;
#pragma unroll 4
    for (int i = l; i < (n >> 3); i += 16) {
      const uint4 a = wr[i];
      const float4 b0 = x4[2 * i], b1 = x4[2 * i + 1];
      const uint32_t dw[4] = {a.x, a.y, a.z, a.w};
      float lo[4], hi[4];
#pragma unroll
      for (int t = 0; t < 4; t++) {
        lo[t] = TYPE == CTHIP_BF16 ? __uint_as_float(dw[t] << 16) : half_bits_to_float((unsigned short)(dw[t] & 0xffff));
        hi[t] = TYPE == CTHIP_BF16 ? __uint_as_float(dw[t] & 0xffff0000u) : half_bits_to_float((unsigned short)(dw[t] >> 16));
      }
      acc = fmaf(lo[0], b0.x, fmaf(hi[0], b0.y, fmaf(lo[1], b0.z, fmaf(hi[1], b0.w, acc))));
      acc = fmaf(lo[2], b1.x, fmaf(hi[2], b1.y, fmaf(lo[3], b1.z, fmaf(hi[3], b1.w, acc))));
    }
  }
  return acc;
}

// a wavefront normalises one latent (R <= 1024); everything is requested before anything is used
__device__ __forceinline__ void latent_norm(const LatentArgs &a, const float *__restrict__ src, float *__restrict__ dst, int lane) {
  float4 x[4], w[4];
  float ss = 0.0f;
#pragma unroll
  for (int k = 0; k < 4; k++) {
    const int e = min(4 * (lane + 64 * k), a.R - 4);
    x[k] = *(const float4 *)(src + e);
    w[k] = *(const float4 *)(a.norm + e);
  }
#pragma unroll
  for (int k = 0; k < 4; k++)
    if (4 * (lane + 64 * k) < a.R) ss = fmaf(x[k].x, x[k].x, fmaf(x[k].y, x[k].y, fmaf(x[k].z, x[k].z, fmaf(x[k].w, x[k].w, ss))));  // padding entries are zero
  const float rstd = 1.0f / sqrtf(wave_sum(ss) / (float)a.r + a.eps);
#pragma unroll
  for (int k = 0; k < 4; k++) {
    const int e = 4 * (lane + 64 * k);
    if (e < a.R) *(float4 *)(dst + e) = make_float4(x[k].x * rstd * w[k].x, x[k].y * rstd * w[k].y, x[k].z * rstd * w[k].z, x[k].w * rstd * w[k].w);
  }
}

__global__ __launch_bounds__(256) void k_latent_append(LatentArgs a, int s, int n) {
  const int t = blockIdx.x * 4 + (threadIdx.x >> 6);
  if (t >= s) return;
  latent_norm(a, a.p + (int64_t)t * a.ldp + (int64_t)a.H * a.DK, a.cache + (int64_t)(n + t) * a.R, threadIdx.x & 63);
}

int launch_latent_append(const LatentArgs &a, int s, int n) {
  if (s <= 0) return 0;
  hipLaunchKernelGGL(k_latent_append, dim3((unsigned)((s + 3) / 4)), dim3(256), 0, state().stream, a, s, n);
  CTHIP_LAUNCH_CHECK();
  return 0;
}

template <int TYPE>
__global__ __launch_bounds__(256) void k_latent_absorb(LatentArgs a, float *__restrict__ qa, const int *__restrict__ pos) {
  const int rows = a.H * a.R;
  if (blockIdx.x == gridDim.x - 1) {
    if (threadIdx.x < 64) latent_norm(a, a.p + (int64_t)a.H * a.DK, a.cache + (int64_t)pos[0] * a.R, threadIdx.x);
    return;
  }
  const int l = threadIdx.x & 15;
  const int row = blockIdx.x * 16 + (threadIdx.x >> 4);  // R is a multiple of 16: a workgroup stays in one head
  const int h = (blockIdx.x * 16) / a.R;
  if (row >= rows) return;
  const float v = row16_sum(row_dot16<TYPE>(a.absorb, row, a.p + h * a.DK, a.DK, l));
  if (l == 0) qa[row] = v * a.scale;
}

// The visible rows are tiles of 16; range r takes tiles r, r + n, ... of n ranges: its first tile does not depend on how many
// rows there are.  A range's record is merged by every workgroup of k_latent_up, so up to four tiles go to a range before
// more than 64 ranges are used (16 heads at position 1900: 32 / 64 ranges 954 / 942 us per step of the 1b shape).
__device__ __forceinline__ int latent_ranges(int T, int most) {
  const int tiles = (T + 15) >> 4;
  return min(tiles, tiles > 256 ? most : min(most, 64));
}

// Workgroup (range, group of 16 heads), four wavefronts.  A tile of 16 cached rows is fetched once, into LDS, a tile ahead.
//   S^T = C Q^T: a wavefront takes every fourth 16-float piece of the latent; lane l feeds C[key l%16] and Q[head l%16] with
//     the four floats 4 (l/16) .. of the piece (the same order on both sides), so it ends up with keys 4 (l/16) + i of head
//     l % 16; the four wavefronts' sums meet in LDS;
//   O^T += C^T P^T: a wavefront owns every fourth 64-float block of the latent; register i of a lane is exactly the
//     probability that matrix instruction i wants from it, and the 16 bytes 4 (l%16) .. of row 4 (l/16) + i of the tile are its
//     operands for four output tiles (tile t: latent entry 64 b + 4 m + t in row m).
constexpr int part_pitch(int R) { return R + 4; }  // a range's record of one head: R sums, maximum, denominator, two unused
template <int NB>  // 256-float blocks of a latent
__global__ __launch_bounds__(256) void k_latent_attend(LatentArgs a, const float *__restrict__ qa, float *__restrict__ part,
                                                       const int *__restrict__ pos, int ranges) {
  extern __shared__ float tiles_lds[];  // two tiles of 16 rows, R + 4 floats apart
  __shared__ float sx[4][4][64];
  const int lane = threadIdx.x & 63, wv = threadIdx.x >> 6, lo = lane & 15, hi = lane >> 4;
  const int range = blockIdx.x, h0 = blockIdx.y * 16, R = a.R, H = a.H, LD = R + 4;
  const int last = a.rows - 1;  // of the cache; rows past the visible ones are masked
  const int np = R >> 4, hq = min(h0 + lo, H - 1);  // heads past the end repeat the last one and are not stored
  constexpr int NP = 4 * NB;                        // pieces per wavefront, at most
  float4 pf[4][NB];  // rows 4 wv .. 4 wv + 3 of the tile that comes next
  auto fetch = [&](int tile) {
#pragma unroll
    for (int r = 0; r < 4; r++) {
      const float *row = a.cache + (int64_t)min(tile * 16 + 4 * wv + r, last) * R;
#pragma unroll
      for (int b = 0; b < NB; b++) pf[r][b] = *(const float4 *)(row + min(4 * (lane + 64 * b), R - 4));
    }
  };
  fetch(range);  // (which tile a range starts with does not depend on the position)
  const int T = pos[0] + 1, tiles = (T + 15) >> 4;
  float4 q[NP];
#pragma unroll
  for (int i = 0; i < NP; i++) {
    const int pc = wv + 4 * i;
    const float4 v = *(const float4 *)(qa + (int64_t)hq * R + 16 * min(pc, np - 1) + 4 * hi);
    q[i] = pc < np ? v : make_float4(0.f, 0.f, 0.f, 0.f);
  }
  const int nr = latent_ranges(T, ranges);  // every one of them holds at least one row
  if (range >= nr) return;
  auto put = [&](int tile, int buf) {  // rows that no token of this sequence has written are zeroed: their weight is zero, their values need not be numbers
#pragma unroll
    for (int r = 0; r < 4; r++) {
      const bool seen = tile * 16 + 4 * wv + r < T;
      float *row = tiles_lds + (buf * 16 + 4 * wv + r) * LD;
#pragma unroll
      for (int b = 0; b < NB; b++) {
        const int e = 4 * (lane + 64 * b);
        if (e < R) *(float4 *)(row + e) = seen ? pf[r][b] : make_float4(0.f, 0.f, 0.f, 0.f);
      }
    }
  };
  v4f_t o[NB][4];
#pragma unroll
  for (int b = 0; b < NB; b++)
#pragma unroll
    for (int t = 0; t < 4; t++) o[b][t] = v4f_t{0.f, 0.f, 0.f, 0.f};
  float m = -INFINITY, L = 0.0f;
  int buf = 0;
  put(range, 0);
  fetch(min(range + nr, tiles - 1));
  __syncthreads();
  for (int tile = range; tile < tiles; tile += nr, buf ^= 1) {
    const int kb = tile * 16;
    const float *Ct = tiles_lds + buf * 16 * LD;
    v4f_t s0 = {0.f, 0.f, 0.f, 0.f}, s1 = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < NP; i++) {
      const float4 kc = *(const float4 *)(Ct + lo * LD + 16 * min(wv + 4 * i, np - 1) + 4 * hi);  // (past the end: times zeros)
      s0 = __builtin_amdgcn_mfma_f32_16x16x4f32(kc.x, q[i].x, s0, 0, 0, 0);
      s1 = __builtin_amdgcn_mfma_f32_16x16x4f32(kc.y, q[i].y, s1, 0, 0, 0);
      s0 = __builtin_amdgcn_mfma_f32_16x16x4f32(kc.z, q[i].z, s0, 0, 0, 0);
      s1 = __builtin_amdgcn_mfma_f32_16x16x4f32(kc.w, q[i].w, s1, 0, 0, 0);
    }
#pragma unroll
    for (int i = 0; i < 4; i++) sx[wv][i][lane] = s0[i] + s1[i];
    __syncthreads();
    float sc[4], top = -INFINITY;
#pragma unroll
    for (int i = 0; i < 4; i++) {
      sc[i] = (sx[0][i][lane] + sx[1][i][lane]) + (sx[2][i][lane] + sx[3][i][lane]);
      if (kb + 4 * hi + i >= T) sc[i] = -INFINITY;
      top = fmaxf(top, sc[i]);
    }
    top = fmaxf(top, __shfl_xor(top, 16, 64));
    top = fmaxf(top, __shfl_xor(top, 32, 64));
    const float m_new = fmaxf(m, top);  // finite: a tile holds at least one visible row
    const float corr = expf(m - m_new);
    float ps = 0.0f;
#pragma unroll
    for (int i = 0; i < 4; i++) {
      sc[i] = expf(sc[i] - m_new);
      ps += sc[i];
    }
    ps += __shfl_xor(ps, 16, 64);
    ps += __shfl_xor(ps, 32, 64);
    L = fmaf(L, corr, ps);
    m = m_new;
#pragma unroll
    for (int b = 0; b < NB; b++) {
      const float *vcol = Ct + 4 * hi * LD + min(64 * (wv + 4 * b) + 4 * lo, R - 4);  // (past the end: results are not stored)
#pragma unroll
      for (int t = 0; t < 4; t++) o[b][t] *= corr;
#pragma unroll
      for (int i = 0; i < 4; i++) {
        const float4 vc = *(const float4 *)(vcol + i * LD);
        o[b][0] = __builtin_amdgcn_mfma_f32_16x16x4f32(vc.x, sc[i], o[b][0], 0, 0, 0);
        o[b][1] = __builtin_amdgcn_mfma_f32_16x16x4f32(vc.y, sc[i], o[b][1], 0, 0, 0);
        o[b][2] = __builtin_amdgcn_mfma_f32_16x16x4f32(vc.z, sc[i], o[b][2], 0, 0, 0);
        o[b][3] = __builtin_amdgcn_mfma_f32_16x16x4f32(vc.w, sc[i], o[b][3], 0, 0, 0);
      }
    }
    if (tile + nr < tiles) {  // (uniform over the workgroup)
      put(tile + nr, buf ^ 1);
      fetch(min(tile + 2 * nr, tiles - 1));
    }
    __syncthreads();
  }
  if (h0 + lo < H) {
    float *dst = part + ((int64_t)range * H + h0 + lo) * part_pitch(R);
#pragma unroll
    for (int b = 0; b < NB; b++)
#pragma unroll
      for (int i = 0; i < 4; i++) {
        const int e = 64 * (wv + 4 * b) + 4 * (4 * hi + i);
        if (e < R) *(float4 *)(dst + e) = make_float4(o[b][0][i], o[b][1][i], o[b][2][i], o[b][3][i]);
      }
    if (wv == 0 && hi == 0) *(float2 *)(dst + R) = make_float2(m, L);
  }
}

// Workgroup (head, share of its value rows): the ranges merged in LDS, then 16 lanes per value row.  The ranges' sums are
// requested before their weights are known; 256 / (R / 4) groups of threads share the ranges.
template <int TYPE>
__global__ __launch_bounds__(256) void k_latent_up(LatentArgs a, const float *__restrict__ part, float *__restrict__ out,
                                                   const int *__restrict__ pos, int ranges) {
  constexpr int AHEAD = 8;
  extern __shared__ float x[];  // the groups' merged latents, R floats each
  __shared__ float wr[kLatentMaxRanges];
  const int h = blockIdx.x, R = a.R, tid = threadIdx.x, l = tid & 15;
  const float *__restrict__ ph = part + (int64_t)h * part_pitch(R);
  const int64_t pitch = (int64_t)a.H * part_pitch(R);
  const int n4 = R >> 2, ng = 256 / n4, grp = tid / n4, col = 4 * (tid - grp * n4);
  float2 ml[2];
#pragma unroll
  for (int k = 0; k < 2; k++) ml[k] = *(const float2 *)(ph + min((tid & 63) + 64 * k, ranges - 1) * pitch + R);
  float4 t[AHEAD];
#pragma unroll
  for (int k = 0; k < AHEAD; k++) t[k] = *(const float4 *)(ph + min(grp + ng * k, ranges - 1) * pitch + col);
  const float sink = a.sink ? a.sink[h] : -INFINITY;
  const int used = latent_ranges(pos[0] + 1, ranges);
  if (tid < 64) {  // the first wavefront: two ranges per lane, their weights in the merged softmax
    const float m0 = tid < used ? ml[0].x : -INFINITY, d0 = tid < used ? ml[0].y : 0.0f;
    const float m1 = tid + 64 < used ? ml[1].x : -INFINITY, d1 = tid + 64 < used ? ml[1].y : 0.0f;
    const float M = fmaxf(wave_max(fmaxf(m0, m1)), sink);
    const float e0 = expf(m0 - M), e1 = expf(m1 - M);
    const float L = wave_sum(e0 * d0 + e1 * d1) + expf(sink - M);  // (every lane takes part in the sum)
    wr[tid] = e0 / L;
    wr[tid + 64] = e1 / L;
  }
  __syncthreads();
  if (grp < ng) {
    float4 acc = make_float4(0.f, 0.f, 0.f, 0.f);
    auto add = [&](int r, const float4 v) {
      if (r >= used) return;  // (what an unused range holds need not be numbers)
      const float c = wr[r];
      acc.x = fmaf(c, v.x, acc.x), acc.y = fmaf(c, v.y, acc.y), acc.z = fmaf(c, v.z, acc.z), acc.w = fmaf(c, v.w, acc.w);
    };
#pragma unroll
    for (int k = 0; k < AHEAD; k++) add(grp + ng * k, t[k]);
    for (int r0 = grp + ng * AHEAD; r0 < used; r0 += ng * AHEAD) {
#pragma unroll
      for (int k = 0; k < AHEAD; k++) t[k] = *(const float4 *)(ph + min(r0 + ng * k, used - 1) * pitch + col);
#pragma unroll
      for (int k = 0; k < AHEAD; k++) add(r0 + ng * k, t[k]);
    }
    *(float4 *)(x + grp * R + col) = acc;
  }
  __syncthreads();
  if (ng > 1) {
    for (int i = tid; i < R; i += 256) {
      float v = x[i];
      for (int g = 1; g < ng; g++) v += x[g * R + i];
      x[i] = v;  // (read by this thread only until the barrier)
    }
    __syncthreads();
  }
  for (int j = blockIdx.y * 16 + (tid >> 4); j < a.DV; j += 16 * gridDim.y) {
    const float v = row16_sum(row_dot16<TYPE>(a.up, (int64_t)h * a.DV + j, x, R, l));
    if (l == 0) out[h * a.DV + j] = a.gated ? v / (1.0f + expf(-a.p[(int64_t)a.H * a.DK + R + h * a.DV + j])) : v;
  }
}

size_t latent_part_floats(int H, int R, int ranges) { return (size_t)ranges * H * part_pitch(R); }

int launch_latent_step(const LatentArgs &a, const LatentWork &w, float *out, const int *pos) {
  hipStream_t st = state().stream;
  const dim3 ga((unsigned)(a.H * a.R / 16 + 1)), gt((unsigned)w.ranges, (unsigned)((a.H + 15) / 16));
  // value rows of a head shared by as many workgroups as fill the compute units
  int shares = state().compute_units / a.H;
  if (shares > a.DV / 16) shares = a.DV / 16;
  const dim3 gu((unsigned)a.H, (unsigned)(shares < 1 ? 1 : shares));
  const size_t lds = sizeof(float) * (size_t)a.R * (256 / (a.R / 4));
  const size_t lds_tiles = sizeof(float) * 2 * 16 * (size_t)(a.R + 4);
  const int nb = (a.R + 255) / 256;
#define ABSORB(T) hipLaunchKernelGGL((k_latent_absorb<T>), ga, dim3(256), 0, st, a, w.qa, pos)
#define UP(T) hipLaunchKernelGGL((k_latent_up<T>), gu, dim3(256), lds, st, a, w.part, out, pos, w.ranges)
  if (a.type == CTHIP_BF16) ABSORB(CTHIP_BF16);
  else if (a.type == CTHIP_F16) ABSORB(CTHIP_F16);
  else ABSORB(CTHIP_F32);
#define ATTEND(N)                                                                                                                       \
  do {                                                                                                                                  \
    static bool granted = false;                                                                                                        \
    if (lds_tiles > 64 * 1024 && !granted) { /* once per kernel: more than the default share of LDS */                                  \
      CTHIP_CHECK(hipFuncSetAttribute((const void *)k_latent_attend<N>, hipFuncAttributeMaxDynamicSharedMemorySize, 140 * 1024));         \
      granted = true;                                                                                                                   \
    }                                                                                                                                   \
    hipLaunchKernelGGL((k_latent_attend<N>), gt, dim3(256), lds_tiles, st, a, w.qa, w.part, pos, w.ranges);                              \
  } while (0)
  if (nb <= 1) ATTEND(1);
  else if (nb <= 2) ATTEND(2);
  else if (nb <= 4) ATTEND(4);
  else return fail(CTHIP_E_UNSUPPORTED, "latent attention: a latent of %d (at most 1024)", a.R);
#undef ATTEND
  if (a.type == CTHIP_BF16) UP(CTHIP_BF16);
  else if (a.type == CTHIP_F16) UP(CTHIP_F16);
  else UP(CTHIP_F32);
#undef ABSORB
#undef UP
  CTHIP_LAUNCH_CHECK();
  return 0;
}

// ------------------------------------------------------------------ small pieces
template <typename T>
__global__ __launch_bounds__(256) void k_place(T *__restrict__ dst, const T *__restrict__ src, int64_t rows, int64_t cols, int64_t r0,
                                               int64_t hr, int64_t hrp, int64_t hc, int64_t hcp, int64_t ld) {
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (i >= rows * cols) return;
  const int64_t r = i / cols, c = i % cols;
  dst[(r0 + (r / hr) * hrp + r % hr) * ld + (c / hc) * hcp + c % hc] = src[i];
}
template <typename T>
__global__ __launch_bounds__(256) void k_place_transposed(T *__restrict__ dst, const T *__restrict__ src, int64_t heads, int64_t hr,
                                                          int64_t hrp, int64_t cols, int64_t colsp) {
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (i >= heads * hr * cols) return;
  const int64_t c = i % cols, r = (i / cols) % hr, h = i / (cols * hr);
  dst[(h * colsp + c) * hrp + r] = src[i];
}
int launch_place(void *dst, const void *src, int es, int64_t rows, int64_t cols, int64_t r0, int64_t hr, int64_t hrp, int64_t hc,
                 int64_t hcp, int64_t ld) {
  const dim3 grid((unsigned)((rows * cols + 255) / 256));
  if (es == 4) hipLaunchKernelGGL((k_place<uint32_t>), grid, dim3(256), 0, state().stream, (uint32_t *)dst, (const uint32_t *)src, rows, cols, r0, hr, hrp, hc, hcp, ld);
  else hipLaunchKernelGGL((k_place<unsigned short>), grid, dim3(256), 0, state().stream, (unsigned short *)dst, (const unsigned short *)src, rows, cols, r0, hr, hrp, hc, hcp, ld);
  CTHIP_LAUNCH_CHECK();
  return 0;
}
int launch_place_transposed(void *dst, const void *src, int es, int64_t heads, int64_t hr, int64_t hrp, int64_t cols, int64_t colsp) {
  const dim3 grid((unsigned)((heads * hr * cols + 255) / 256));
  if (es == 4) hipLaunchKernelGGL((k_place_transposed<uint32_t>), grid, dim3(256), 0, state().stream, (uint32_t *)dst, (const uint32_t *)src, heads, hr, hrp, cols, colsp);
  else hipLaunchKernelGGL((k_place_transposed<unsigned short>), grid, dim3(256), 0, state().stream, (unsigned short *)dst, (const unsigned short *)src, heads, hr, hrp, cols, colsp);
  CTHIP_LAUNCH_CHECK();
  return 0;
}

// built once per session, in double precision: an angle of thousands of radians keeps its last digits
__global__ __launch_bounds__(256) void k_sinusoid_table(float *__restrict__ table, int64_t n, int dim, double base) {
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (i >= n) return;
  const int d = (int)(i % dim);
  const double angle = (double)(i / dim) * pow(base, -(double)(d & ~1) / (double)dim);
  table[i] = (float)((d & 1) ? cos(angle) : sin(angle));
}
int launch_sinusoid_table(float *table, int rows, int dim, double base) {
  const int64_t n = (int64_t)rows * dim;
  hipLaunchKernelGGL(k_sinusoid_table, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, state().stream, table, n, dim, base);
  CTHIP_LAUNCH_CHECK();
  return 0;
}

__global__ __launch_bounds__(256) void k_place_taps(float *__restrict__ dst, const float *__restrict__ w, int channels, int taps, int C,
                                                    int ch0, int hr, int hrp) {
  const int i = blockIdx.x * 256 + threadIdx.x;
  if (i >= channels * taps) return;
  const int c = i / taps, t = i % taps;
  dst[(int64_t)(taps - 1 - t) * C + ch0 + (c / hr) * hrp + c % hr] = w[i];
}
int launch_place_taps(float *dst, const float *w, int channels, int taps, int C, int ch0, int hr, int hrp) {
  hipLaunchKernelGGL(k_place_taps, dim3((unsigned)((channels * taps + 255) / 256)), dim3(256), 0, state().stream, dst, w, channels, taps, C, ch0, hr, hrp);
  CTHIP_LAUNCH_CHECK();
  return 0;
}

__global__ __launch_bounds__(256) void k_neg_exp(float *__restrict__ y, const float *__restrict__ x, int n) {
  const int i = blockIdx.x * 256 + threadIdx.x;
  if (i < n) y[i] = -expf(x[i]);
}
int launch_neg_exp(float *y, const float *x, int n) {
  hipLaunchKernelGGL(k_neg_exp, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, state().stream, y, x, n);
  CTHIP_LAUNCH_CHECK();
  return 0;
}

__global__ __launch_bounds__(256) void k_softcap(float *__restrict__ y, int64_t n, float cap) {
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (i < n) y[i] = softcap(y[i], cap);
}
int launch_softcap(float *y, int64_t n, float cap) {
  if (n <= 0) return 0;
  hipLaunchKernelGGL(k_softcap, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, state().stream, y, n, cap);
  CTHIP_LAUNCH_CHECK();
  return 0;
}

__global__ __launch_bounds__(256) void k_gather_rows(float *__restrict__ dst, const float *__restrict__ src, const int *__restrict__ rows, int n) {
  const float *s = src + (int64_t)rows[blockIdx.x] * n;
  for (int i = threadIdx.x; i < n; i += 256) dst[(int64_t)blockIdx.x * n + i] = s[i];
}
int launch_gather_rows(float *dst, const float *src, const int *rows, int nrows, int n) {
  if (nrows <= 0) return 0;
  hipLaunchKernelGGL(k_gather_rows, dim3((unsigned)nrows), dim3(256), 0, state().stream, dst, src, rows, n);
  CTHIP_LAUNCH_CHECK();
  return 0;
}

}  // namespace cthip
