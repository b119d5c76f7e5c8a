// Lightning attention: per head a matrix state S (key dimension x value dimension, fp32) with a fixed decay,
//   S <- decay S + k v^T,   o = S^T q,
// q, k and v behind silu.  The concatenated heads of a token are divided by their root mean square, weighted and multiplied
// by the sigmoid of a gate.  The state is kept as [head][value column][key].  Decode steps are parallel.hip's.
//
// Prompts, in chunks of 64 tokens (L of them in the last one).  The decay does not depend on the tokens, so nothing but the
// states has to go from chunk to chunk in order:
//   k_lightning_local   U_c = sum_j decay^(L - 1 - j) k_j v_j^T, every chunk and head by itself
//   k_lightning_carry   S_c = the state in front of chunk c: S_(c+1) = decay^L S_c + U_c, every element by itself
//   k_lightning_out     o_i = decay^(i + 1) S_c^T q_i + sum_(j <= i) decay^(i - j) (q_i . k_j) v_j, every chunk and head by itself
// on v_mfma_f32_16x16x4_f32 (fp32 products).  Operand order as in delta.hip: lane l supplies a row's four floats 4 (l/16) ..
// of a 16-float piece to four matrix instructions, and a result tile holds rows 4 (l/16) + i of column l % 16 in register i.
#include "common.h"
#include "mixers.h"

namespace cthip {

constexpr int kLightChunk = 64;
constexpr int kLightSegment = 64;  // chunks whose states are held at a time
typedef float v4f_t __attribute__((ext_vector_type(4)));

__device__ __forceinline__ v4f_t mfma4(const float4 a, const v4f_t b, v4f_t c) {
  c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.x, b[0], c, 0, 0, 0);
  c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.y, b[1], c, 0, 0, 0);
  c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.z, b[2], c, 0, 0, 0);
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a.w, b[3], c, 0, 0, 0);
}
__device__ __forceinline__ v4f_t vec4(const float4 a) { return v4f_t{a.x, a.y, a.z, a.w}; }

// q, k and v of every row pass silu in place
__global__ __launch_bounds__(256) void k_lightning_silu(float *__restrict__ p, int64_t ldp, int w) {
  const int e = 4 * (blockIdx.y * 256 + threadIdx.x);
  if (e >= w) return;
  float4 *x = (float4 *)(p + (int64_t)blockIdx.x * ldp + e);
  const float4 v = *x;
  *x = make_float4(ct_silu(v.x), ct_silu(v.y), ct_silu(v.z), ct_silu(v.w));
}

// Workgroup (chunk, head); wavefront w takes the key tiles w, w + 4, ... against every value tile.
template <int NV>  // 16-column value tiles, at most
__global__ __launch_bounds__(256) void k_lightning_local(LightningArgs a, const float *__restrict__ p, float *__restrict__ U, int s) {
  const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6, lo = lane & 15, hi = lane >> 4;
  const int c0 = blockIdx.x * kLightChunk, h = blockIdx.y, DK = a.DK, DV = a.DV, nv = DV >> 4;
  const int last = min(c0 + kLightChunk, s) - 1;
  const float lg = a.decay[a.H + h];
  const float *__restrict__ K = p + (int64_t)(a.H + h) * DK, *__restrict__ V = p + 2 * (int64_t)a.H * DK + (int64_t)h * DV;
  float *__restrict__ Uh = U + ((int64_t)blockIdx.x * a.H + h) * DV * DK;
  for (int kt = wv; kt < (DK >> 4); kt += 4) {
    v4f_t acc[NV];
#pragma unroll
    for (int v = 0; v < NV; v++) acc[v] = v4f_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (int j = 0; j < kLightChunk; j += 4) {  // lane (lo, hi): token j + hi
      const int t = c0 + j + hi, tc = min(t, last);
      const float w = t <= last ? exp2f((float)(last - t) * lg) : 0.0f;
      const float kx = K[(int64_t)tc * a.ldp + 16 * kt + lo] * w;
#pragma unroll
      for (int v = 0; v < NV; v++)
        acc[v] = __builtin_amdgcn_mfma_f32_16x16x4f32(kx, V[(int64_t)tc * a.ldp + 16 * min(v, nv - 1) + lo], acc[v], 0, 0, 0);
    }
#pragma unroll
    for (int v = 0; v < NV; v++)
      if (v < nv) *(v4f_t *)(Uh + (int64_t)(16 * v + lo) * DK + 16 * kt + 4 * hi) = acc[v];
  }
}

// four elements of the state per thread: U_c is replaced by the state in front of chunk c, S by the one behind the last
__global__ __launch_bounds__(256) void k_lightning_carry(LightningArgs a, float *__restrict__ U, int s, int n) {
  constexpr int AHEAD = 8;
  const int64_t e4 = (int64_t)blockIdx.x * 256 + threadIdx.x, total = (int64_t)a.H * a.DV * a.DK / 4;
  if (e4 >= total) return;
  const int h = (int)(e4 / ((int64_t)a.DV * a.DK / 4)), nch = (s + kLightChunk - 1) / kLightChunk;
  const float lg = a.decay[a.H + h], full = exp2f((float)kLightChunk * lg), rest = exp2f((float)(s - (nch - 1) * kLightChunk) * lg);
  float4 S = n > 0 ? ((const float4 *)a.S)[e4] : make_float4(0.f, 0.f, 0.f, 0.f);
  float4 *__restrict__ Ue = (float4 *)U + e4;
  for (int c0 = 0; c0 < nch; c0 += AHEAD) {
    float4 u[AHEAD];
#pragma unroll
    for (int k = 0; k < AHEAD; k++) u[k] = Ue[(int64_t)min(c0 + k, nch - 1) * total];
#pragma unroll
    for (int k = 0; k < AHEAD; k++) {
      if (c0 + k >= nch) break;
      Ue[(int64_t)(c0 + k) * total] = S;
      const float g = c0 + k == nch - 1 ? rest : full;
      S = make_float4(fmaf(S.x, g, u[k].x), fmaf(S.y, g, u[k].y), fmaf(S.z, g, u[k].z), fmaf(S.w, g, u[k].w));
    }
  }
  ((float4 *)a.S)[e4] = S;
}

// Workgroup (chunk, head); wavefront w owns the chunk's rows 16 w .. 16 w + 15.
template <int NK>  // 16-entry pieces of a key, at most
__global__ __launch_bounds__(256) void k_lightning_out(LightningArgs a, const float *__restrict__ p, const float *__restrict__ U, float *__restrict__ out,
                                                       int64_t ldo, int s) {
  const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6, lo = lane & 15, hi = lane >> 4;
  const int c0 = blockIdx.x * kLightChunk, h = blockIdx.y, DK = a.DK, DV = a.DV, nk = DK >> 4;
  if (c0 + 16 * wv >= s) return;
  const float lg = a.decay[a.H + h];
  const float *__restrict__ Q = p + (int64_t)h * DK, *__restrict__ K = p + (int64_t)(a.H + h) * DK;
  const float *__restrict__ V = p + 2 * (int64_t)a.H * DK + (int64_t)h * DV;
  const float *__restrict__ S = U + ((int64_t)blockIdx.x * a.H + h) * DV * DK;
  auto row = [&](int i) { return (int64_t)min(c0 + i, s - 1) * a.ldp; };  // rows past the end repeat the last one: later than every stored row
  float4 q[NK];
#pragma unroll
  for (int c = 0; c < NK; c++) {
    q[c] = *(const float4 *)(Q + row(16 * wv + lo) + 16 * min(c, nk - 1) + 4 * hi);
    if (c >= nk) q[c] = make_float4(0.f, 0.f, 0.f, 0.f);
  }
  // P[kt]: register t = key 16 kt + 4 hi + t of query lo
  float4 P[4];
#pragma unroll
  for (int kt = 0; kt < 4; kt++) {
    P[kt] = make_float4(0.f, 0.f, 0.f, 0.f);
    if (kt > wv) continue;  // (uniform)
    v4f_t acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int c = 0; c < NK; c++) acc = mfma4(*(const float4 *)(K + row(16 * kt + lo) + 16 * min(c, nk - 1) + 4 * hi), vec4(q[c]), acc);
    float w[4];
#pragma unroll
    for (int t = 0; t < 4; t++) {
      const int d = 16 * (wv - kt) + lo - 4 * hi - t;
      w[t] = d >= 0 ? acc[t] * exp2f((float)d * lg) : 0.0f;
    }
    P[kt] = make_float4(w[0], w[1], w[2], w[3]);
  }
  float g[4];
#pragma unroll
  for (int t = 0; t < 4; t++) g[t] = exp2f((float)(16 * wv + 4 * hi + t + 1) * lg);
  for (int vt = 0; vt < (DV >> 4); vt++) {
    const float *sr = S + (int64_t)(16 * vt + lo) * DK + 4 * hi;
    v4f_t o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int c = 0; c < NK; c++) o = mfma4(q[c], vec4(*(const float4 *)(sr + 16 * min(c, nk - 1))), o);
#pragma unroll
    for (int t = 0; t < 4; t++) o[t] *= g[t];
#pragma unroll
    for (int kt = 0; kt < 4; kt++) {
      if (kt > wv) continue;
      v4f_t v;
#pragma unroll
      for (int t = 0; t < 4; t++) v[t] = V[row(16 * kt + 4 * hi + t) + 16 * vt + lo];
      o = mfma4(P[kt], v, o);
    }
#pragma unroll
    for (int t = 0; t < 4; t++) {
      const int i = c0 + 16 * wv + 4 * hi + t;
      if (i < s) out[(int64_t)i * ldo + (int64_t)h * DV + 16 * vt + lo] = o[t];
    }
  }
}

// a workgroup per token: out <- out / rms(out) * norm * sigmoid(gate) * out_scale
__global__ __launch_bounds__(256) void k_lightning_finish(LightningArgs a, const float *__restrict__ p, float *__restrict__ out, int64_t ldo) {
  __shared__ float red[4];
  const int tid = threadIdx.x, W = a.H * a.DV;
  float *__restrict__ o = out + (int64_t)blockIdx.x * ldo;
  const float *__restrict__ g = p + (int64_t)blockIdx.x * a.ldp + (int64_t)a.H * (2 * a.DK + a.DV);
  float ss = 0.0f;
  for (int e = 4 * tid; e < W; e += 1024) {
    const float4 x = *(const float4 *)(o + e);
    ss = fmaf(x.x, x.x, fmaf(x.y, x.y, fmaf(x.z, x.z, fmaf(x.w, x.w, ss))));
  }
  ss = wave_sum(ss);
  if ((tid & 63) == 0) red[tid >> 6] = ss;
  __syncthreads();
  const float rstd = a.out_scale / sqrtf(((red[0] + red[1]) + (red[2] + red[3])) / (float)(a.H * a.dv) + a.eps);
  for (int e = 4 * tid; e < W; e += 1024) {
    const float4 x = *(const float4 *)(o + e), w = *(const float4 *)(a.norm + e), z = *(const float4 *)(g + e);
    *(float4 *)(o + e) = make_float4(x.x * rstd * w.x * ct_sigmoid(z.x), x.y * rstd * w.y * ct_sigmoid(z.y), x.z * rstd * w.z * ct_sigmoid(z.z),
                                     x.w * rstd * w.w * ct_sigmoid(z.w));
  }
}

size_t lightning_scratch_floats(const LightningArgs &a, int s) {
  int chunks = (s + kLightChunk - 1) / kLightChunk;
  if (chunks > kLightSegment) chunks = kLightSegment;
  return (size_t)chunks * a.H * a.DV * a.DK;
}

int launch_lightning_rows(const LightningArgs &a, float *p, float *out, int64_t ldo, int s, int n, float *scratch) {
  if (s <= 0) return 0;
  if (a.DK > 256 || a.DV > 256) return fail(CTHIP_E_UNSUPPORTED, "lightning attention: heads of %d / %d (at most 256)", a.DK, a.DV);
  hipStream_t st = state().stream;
  const dim3 b256(256);
  const int w = a.H * (2 * a.DK + a.DV);
  hipLaunchKernelGGL(k_lightning_silu, dim3((unsigned)s, (unsigned)((w / 4 + 255) / 256)), b256, 0, st, p, a.ldp, w);
  const int64_t quads = (int64_t)a.H * a.DV * a.DK / 4;
  for (int t0 = 0; t0 < s; t0 += kLightChunk * kLightSegment) {
    const int m = s - t0 < kLightChunk * kLightSegment ? s - t0 : kLightChunk * kLightSegment;
    float *pt = p + (int64_t)t0 * a.ldp, *ot = out + (int64_t)t0 * ldo;
    const dim3 grid((unsigned)((m + kLightChunk - 1) / kLightChunk), (unsigned)a.H);
#define LOCAL(N) hipLaunchKernelGGL((k_lightning_local<N>), grid, b256, 0, st, a, pt, scratch, m)
#define OUT(N) hipLaunchKernelGGL((k_lightning_out<N>), grid, b256, 0, st, a, pt, scratch, ot, ldo, m)
    if (a.DV <= 32) LOCAL(2);
    else if (a.DV <= 64) LOCAL(4);
    else if (a.DV <= 128) LOCAL(8);
    else LOCAL(16);
    hipLaunchKernelGGL(k_lightning_carry, dim3((unsigned)((quads + 255) / 256)), b256, 0, st, a, scratch, m, n + t0);
    if (a.DK <= 32) OUT(2);
    else if (a.DK <= 64) OUT(4);
    else if (a.DK <= 128) OUT(8);
    else OUT(16);
#undef LOCAL
#undef OUT
    CTHIP_LAUNCH_CHECK();
  }
  hipLaunchKernelGGL(k_lightning_finish, dim3((unsigned)s), b256, 0, st, a, p, out, ldo);
  CTHIP_LAUNCH_CHECK();
  return 0;
}

}  // namespace cthip
