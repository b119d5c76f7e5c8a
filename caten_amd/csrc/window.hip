// Attention over a sliding window: grouped-query heads, keys j of position i with 0 <= i - j < window.  Queries and keys
// may pass an RMS norm over the whole projection (all heads at once) and a rotation of their first 2 x half entries
// (entries i and i + half of a head are a pair; cosines and sines come from a table); the softmax may have a sink; the
// concatenated heads may be multiplied by the sigmoid of a gate.
//
// The cache is a pair of rings: the token at position i leaves its normalised, rotated key and its value in row i mod rows,
// rows = min(window, longest sequence), so a row is overwritten by the first position that does not see it any more.
//
// Decode steps are parallel.hip's.  Prompts: k_window_prepare lines the visible earlier rows and the portion's own rows up
// (queries are normalised and rotated in place), attn_rows.h attends over them, k_window_keep refills the rings.
#include "common.h"
#include "mixers.h"

namespace cthip {

int window_prev(const WindowArgs &a, int n) { return n < a.window - 1 ? n : a.window - 1; }

// Workgroup t < s: token n + t.  Workgroups s + r: the ring row of position n - prev + r.
__global__ __launch_bounds__(256) void k_window_prepare(WindowArgs a, float *__restrict__ p, float *__restrict__ kbuf, float *__restrict__ vbuf,
                                                        int s, int n, int prev) {
  __shared__ float red[8];
  const int tid = threadIdx.x, KW = a.G * a.DK, VW = a.G * a.DV, QW = a.H * a.DK;
  if ((int)blockIdx.x >= s) {
    const int r = blockIdx.x - s, slot = (n - prev + r) % a.rows;
    for (int e = 4 * tid; e < KW; e += 1024) *(float4 *)(kbuf + (int64_t)r * KW + e) = *(const float4 *)(a.K + (int64_t)slot * KW + e);
    for (int e = 4 * tid; e < VW; e += 1024) *(float4 *)(vbuf + (int64_t)r * VW + e) = *(const float4 *)(a.V + (int64_t)slot * VW + e);
    return;
  }
  const int t = blockIdx.x;
  float *__restrict__ q = p + (int64_t)t * a.ldp;
  const float *__restrict__ k = q + QW, *__restrict__ v = k + KW;
  float *__restrict__ kd = kbuf + (int64_t)(prev + t) * KW, *__restrict__ vd = vbuf + (int64_t)(prev + t) * VW;
  for (int e = 4 * tid; e < VW; e += 1024) *(float4 *)(vd + e) = *(const float4 *)(v + e);
  float qs = 1.0f, ks = 1.0f;
  if (a.qnorm) {  // (padding entries are zero)
    float sq = 0.0f, sk = 0.0f;
    for (int e = 4 * tid; e < QW; e += 1024) {
      const float4 x = *(const float4 *)(q + e);
      sq = fmaf(x.x, x.x, fmaf(x.y, x.y, fmaf(x.z, x.z, fmaf(x.w, x.w, sq))));
    }
    for (int e = 4 * tid; e < KW; e += 1024) {
      const float4 x = *(const float4 *)(k + e);
      sk = fmaf(x.x, x.x, fmaf(x.y, x.y, fmaf(x.z, x.z, fmaf(x.w, x.w, sk))));
    }
    sq = wave_sum(sq), sk = wave_sum(sk);
    if ((tid & 63) == 0) red[tid >> 6] = sq, red[4 + (tid >> 6)] = sk;
    __syncthreads();
    qs = 1.0f / sqrtf(((red[0] + red[1]) + (red[2] + red[3])) / (float)(a.H * a.dk) + a.eps);
    ks = 1.0f / sqrtf(((red[4] + red[5]) + (red[6] + red[7])) / (float)(a.G * a.dk) + a.eps);
  }
  const float2 *__restrict__ cs = a.rope ? a.rope + (int64_t)(n + t) * a.half : nullptr;
  const int half = a.rope ? a.half : 0, per = a.DK - half;  // items of a head: its pairs, then its unpaired entries
  auto turn = [&](const float *src, float *dst, const float *w, float rstd, int heads) {
    for (int it = tid; it < heads * per; it += 256) {
      const int h = it / per, i = it - h * per, e = h * a.DK + (i < half ? i : i + half);
      const float x0 = src[e] * rstd * (w ? w[e] : 1.0f);
      if (i < half) {
        const float x1 = src[e + half] * rstd * (w ? w[e + half] : 1.0f);
        const float2 c = cs[i];
        float o0, o1;
        rope_pair(x0, x1, c.y, c.x, o0, o1);
        dst[e] = o0;
        dst[e + half] = o1;
      } else {
        dst[e] = x0;
      }
    }
  };
  turn(q, q, a.qnorm, qs, a.H);
  turn(k, kd, a.knorm, ks, a.G);
}

int launch_window_prepare(const WindowArgs &a, float *p, float *kbuf, float *vbuf, int s, int n) {
  if (s <= 0) return 0;
  const int prev = window_prev(a, n);
  hipLaunchKernelGGL(k_window_prepare, dim3((unsigned)(s + prev)), dim3(256), 0, state().stream, a, p, kbuf, vbuf, s, n, prev);
  CTHIP_LAUNCH_CHECK();
  return 0;
}

__global__ __launch_bounds__(256) void k_window_keep(WindowArgs a, const float *__restrict__ kbuf, const float *__restrict__ vbuf, int s, int n,
                                                     int prev) {
  const int t = s - 1 - (int)blockIdx.x, tid = threadIdx.x, KW = a.G * a.DK, VW = a.G * a.DV;
  const int slot = (n + t) % a.rows;
  for (int e = 4 * tid; e < KW; e += 1024) *(float4 *)(a.K + (int64_t)slot * KW + e) = *(const float4 *)(kbuf + (int64_t)(prev + t) * KW + e);
  for (int e = 4 * tid; e < VW; e += 1024) *(float4 *)(a.V + (int64_t)slot * VW + e) = *(const float4 *)(vbuf + (int64_t)(prev + t) * VW + e);
}
int launch_window_keep(const WindowArgs &a, const float *kbuf, const float *vbuf, int s, int n) {
  if (s <= 0) return 0;
  hipLaunchKernelGGL(k_window_keep, dim3((unsigned)(s < a.rows ? s : a.rows)), dim3(256), 0, state().stream, a, kbuf, vbuf, s, n, window_prev(a, n));
  CTHIP_LAUNCH_CHECK();
  return 0;
}

// ------------------------------------------------------------------ small pieces
// built once per session, in double precision: an angle of thousands of radians keeps its last digits
__global__ __launch_bounds__(256) void k_rope_table(float2 *__restrict__ table, const double *__restrict__ freqs, int64_t n, int half, double mscale) {
  const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (i >= n) return;
  const double angle = (double)(i / half) * freqs[i % half];
  table[i] = make_float2((float)(cos(angle) * mscale), (float)(sin(angle) * mscale));
}
int launch_rope_table(float2 *table, const double *freqs, int rows, int half, double mscale) {
  const int64_t n = (int64_t)rows * half;
  if (n <= 0) return 0;
  hipLaunchKernelGGL(k_rope_table, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, state().stream, table, freqs, n, half, mscale);
  CTHIP_LAUNCH_CHECK();
  return 0;
}

__global__ __launch_bounds__(256) void k_add_one(float *__restrict__ x, int n) {
  const int i = blockIdx.x * 256 + threadIdx.x;
  if (i < n) x[i] += 1.0f;
}
int launch_add_one(float *x, int n) {
  hipLaunchKernelGGL(k_add_one, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, state().stream, x, n);
  CTHIP_LAUNCH_CHECK();
  return 0;
}

__global__ __launch_bounds__(256) void k_add_embedding(float *__restrict__ x, const float *__restrict__ wte, const float *__restrict__ wpe,
                                                       const int *__restrict__ ids, const int *__restrict__ pos, int vocab, int n, int max_pos) {
  const int i = blockIdx.y * 256 + threadIdx.x, id = ids[blockIdx.x];
  if (i >= n) return;
  float v = id >= 0 && id < vocab ? wte[(int64_t)id * n + i] : 0.0f;
  if (wpe) {
    const int p = pos[0] + (int)blockIdx.x;
    v += p >= 0 && p < max_pos ? wpe[(int64_t)p * n + i] : 0.0f;
  }
  x[(int64_t)blockIdx.x * n + i] += v;
}
int launch_add_embedding(float *x, const float *wte, const float *wpe, const int *ids, const int *pos, int ntok, int vocab, int n, int max_pos) {
  if (ntok <= 0) return 0;
  hipLaunchKernelGGL(k_add_embedding, dim3((unsigned)ntok, (unsigned)((n + 255) / 256)), dim3(256), 0, state().stream, x, wte, wpe, ids, pos, vocab, n, max_pos);
  CTHIP_LAUNCH_CHECK();
  return 0;
}

}  // namespace cthip
