// Gated delta rule: per head a matrix state S (key dimension x value dimension, fp32) that every token decays,
// corrects towards its value along its key and reads with its query:
//   S <- g S,   u = beta (v - S^T k),   S <- S + k u^T,   o = S^T q.
// q, k and v have passed a short causal convolution and silu; q and k are unit vectors (q also scaled by dk^(-1/2));
// g = exp(-exp(A_log) softplus(a + dt_bias)) and beta = sigmoid(b) are one number per head and token.  A head's output is
// divided by its root mean square, weighted, and multiplied by silu of its gate.
//
// The state is kept as [head][value column][key], so that the 16 lanes that own a value column read its keys as
// consecutive 16-byte pieces and both sums over the keys (S^T k, S^T q) are DPP additions inside a row of lanes.
//
//   decode   one launch: a workgroup per head, 16 lanes per value column, the whole state in registers between its one
//            read and its one write;
//   prompts  k_delta_prep (convolutions, unit vectors, gates, one workgroup per token), the recurrence
//            (k_delta_scan token by token, or chunk by chunk on the matrix cores, see below), k_delta_finish (norm and
//            gate), k_delta_history.
//
// The history is a ring of `taps` raw projection rows: a token at position i writes slot i mod taps and reads the
// taps - 1 others, so a launch never reads a slot that it writes.
#include "common.h"
#include "mixers.h"

namespace cthip {

__device__ __forceinline__ float delta_silu(float z) { return z / (1.0f + expf(-z)); }
__device__ __forceinline__ float delta_log_decay(float neg_a, float z) {  // log g
  return neg_a * (fmaxf(z, 0.0f) + log1pf(expf(-fabsf(z))));
}

// one token per launch
template <int NC, int CPG>
__global__ __launch_bounds__(1024) void k_delta_step(DeltaArgs a, float *__restrict__ out, const int *__restrict__ tokpos,
                                                     const int *__restrict__ ctrl) {
  extern __shared__ float os[];  // DV outputs of the head, then 16 partial sums
  float *red = os + a.DV;
  const int tid = threadIdx.x, l = tid & 15, grp = tid >> 4, ngrp = blockDim.x >> 4;
  const int h = blockIdx.x, rep = a.H / a.KH, kh = h / rep;
  const int DK = a.DK, DV = a.DV, C = a.C, taps = a.taps;
  float *__restrict__ Sh = a.S + (int64_t)h * DV * DK;
  // the state first: nothing else is needed to ask for it
  float4 s[CPG][NC];
  auto load_state = [&](int c0) {
#pragma unroll
    for (int k = 0; k < CPG; k++) {
      const int c = min(c0 + grp + ngrp * k, DV - 1);
#pragma unroll
      for (int i = 0; i < NC; i++) {
        const int e = min(4 * (l + 16 * i), DK - 4);  // pieces past the end repeat the last one: their keys are zero
        s[k][i] = *(const float4 *)(Sh + (int64_t)c * DK + e);
      }
    }
  };
  load_state(0);
  const int pos = tokpos[1];
  const bool ended = ctrl && ctrl[1] != 0;
  const float *__restrict__ p = a.p;
  const int qo = kh * DK, ko = a.KH * DK + kh * DK, vo = 2 * a.KH * DK + h * DV, go = C + h * DV, bo = C + a.H * DV + h;
  const int slot = pos % taps;
  auto back = [&](int j) { int t = slot - j; return t < 0 ? t + taps : t; };  // slot of the token j steps back (j < taps)
  auto conv4 = [&](int ch) {
    float4 x = *(const float4 *)(p + ch), w = *(const float4 *)(a.conv + ch);
    float4 r = make_float4(x.x * w.x, x.y * w.y, x.z * w.z, x.w * w.w);
    const int nb = min(taps - 1, pos);
    for (int j = 1; j <= nb; j++) {
      x = *(const float4 *)(a.ring + (int64_t)back(j) * C + ch);
      w = *(const float4 *)(a.conv + (int64_t)j * C + ch);
      r.x = fmaf(x.x, w.x, r.x), r.y = fmaf(x.y, w.y, r.y), r.z = fmaf(x.z, w.z, r.z), r.w = fmaf(x.w, w.w, r.w);
    }
    return make_float4(delta_silu(r.x), delta_silu(r.y), delta_silu(r.z), delta_silu(r.w));
  };
  auto conv1 = [&](int ch) {
    float r = p[ch] * a.conv[ch];
    const int nb = min(taps - 1, pos);
    for (int j = 1; j <= nb; j++) r = fmaf(a.ring[(int64_t)back(j) * C + ch], a.conv[(int64_t)j * C + ch], r);
    return delta_silu(r);
  };
  float4 q[NC], k[NC];
  float qq = 0.0f, kk = 0.0f;
#pragma unroll
  for (int i = 0; i < NC; i++) {
    const int e = 4 * (l + 16 * i);
    q[i] = k[i] = make_float4(0.f, 0.f, 0.f, 0.f);
    if (e < DK) {
      q[i] = conv4(qo + e);
      k[i] = conv4(ko + e);
    }
    qq += q[i].x * q[i].x + q[i].y * q[i].y + q[i].z * q[i].z + q[i].w * q[i].w;
    kk += k[i].x * k[i].x + k[i].y * k[i].y + k[i].z * k[i].z + k[i].w * k[i].w;
  }
  const float qs = 1.0f / (sqrtf(row16_sum(qq) + 1e-6f) * sqrtf((float)a.dk)), ks = 1.0f / sqrtf(row16_sum(kk) + 1e-6f);
#pragma unroll
  for (int i = 0; i < NC; i++) {
    q[i].x *= qs, q[i].y *= qs, q[i].z *= qs, q[i].w *= qs;
    k[i].x *= ks, k[i].y *= ks, k[i].z *= ks, k[i].w *= ks;
  }
  const float beta = 1.0f / (1.0f + expf(-p[bo]));
  const float g = pos == 0 ? 0.0f : expf(delta_log_decay(a.neg_a[h], p[bo + a.H] + a.dt_bias[h]));  // a sequence starts from zero
  float o2 = 0.0f;
  for (int c0 = 0; c0 < DV; c0 += ngrp * CPG) {
    if (c0 > 0) load_state(c0);
#pragma unroll
    for (int kc = 0; kc < CPG; kc++) {
      const int c = c0 + grp + ngrp * kc;
      const bool in = c < DV;
      const float v = conv1(vo + (in ? c : 0));
      float dot = 0.0f;
#pragma unroll
      for (int i = 0; i < NC; i++) {
        float4 &t = s[kc][i];
        if (pos == 0) t = make_float4(0.f, 0.f, 0.f, 0.f);  // (whatever an earlier sequence left, also no number)
        t.x *= g, t.y *= g, t.z *= g, t.w *= g;
        dot = fmaf(t.x, k[i].x, fmaf(t.y, k[i].y, fmaf(t.z, k[i].z, fmaf(t.w, k[i].w, dot))));
      }
      const float u = beta * (v - row16_sum(dot));
      float o = 0.0f;
#pragma unroll
      for (int i = 0; i < NC; i++) {
        float4 &t = s[kc][i];
        t.x = fmaf(k[i].x, u, t.x), t.y = fmaf(k[i].y, u, t.y), t.z = fmaf(k[i].z, u, t.z), t.w = fmaf(k[i].w, u, t.w);
        o = fmaf(t.x, q[i].x, fmaf(t.y, q[i].y, fmaf(t.z, q[i].z, fmaf(t.w, q[i].w, o))));
        const int e = 4 * (l + 16 * i);
        if (in && e < DK && !ended) *(float4 *)(Sh + (int64_t)c * DK + e) = t;
      }
      o = row16_sum(o);
      if (in && l == 0) {
        os[c] = o;
        o2 = fmaf(o, o, o2);
        if (!ended) a.ring[(int64_t)slot * C + vo + c] = p[vo + c];
      }
    }
  }
  if (grp == 0 && h % rep == 0 && !ended) {  // the key head's raw rows, once per group of heads
#pragma unroll
    for (int i = 0; i < NC; i++) {
      const int e = 4 * (l + 16 * i);
      if (e < DK) {
        *(float4 *)(a.ring + (int64_t)slot * C + qo + e) = *(const float4 *)(p + qo + e);
        *(float4 *)(a.ring + (int64_t)slot * C + ko + e) = *(const float4 *)(p + ko + e);
      }
    }
  }
  o2 = wave_sum(o2);
  if ((tid & 63) == 0) red[tid >> 6] = o2;
  __syncthreads();
  float sum = 0.0f;
  for (int w = 0; w < (int)((blockDim.x + 63) >> 6); w++) sum += red[w];
  const float rstd = 1.0f / sqrtf(sum / (float)a.dv + a.eps);
  for (int c = tid; c < DV; c += blockDim.x) out[(int64_t)h * DV + c] = os[c] * rstd * a.norm[c] * delta_silu(p[go + c]);
}

int launch_delta_step(const DeltaArgs &a, float *out, const int *tokpos, const int *ctrl) {
  // 16 lanes per value column, whole wavefronts
  int block = 16 * a.DV;
  if (block > 1024) block = 1024;
  block = (block + 63) & ~63;
  const size_t lds = sizeof(float) * (size_t)(a.DV + 16);
  const int nc = (a.DK + 63) / 64, cpg = (a.DV + block / 16 - 1) / (block / 16);
  dim3 grid(a.H), blk(block);
  hipStream_t st = state().stream;
#define GO(N, K) hipLaunchKernelGGL((k_delta_step<N, K>), grid, blk, lds, st, a, out, tokpos, ctrl)
#define GO_N(N)           \
  if (cpg <= 1) GO(N, 1); \
  else if (cpg <= 2 || N > 2) GO(N, 2); \
  else GO(N, 4)
  if (nc <= 1) { GO_N(1); }
  else if (nc <= 2) { GO_N(2); }
  else if (nc <= 4) { GO_N(4); }
  else return fail(CTHIP_E_UNSUPPORTED, "delta rule: key heads of %d (at most 256)", a.DK);
#undef GO_N
#undef GO
  CTHIP_LAUNCH_CHECK();
  return 0;
}

// ---- prompts ----
struct DeltaRows {
  float *Q, *K, *V, *LG, *BT;  // (s, KH x DK) twice, (s, H x DV), (s, H) twice
};

// a workgroup per token: convolutions, unit vectors, decays' logarithms and step sizes
template <int NC>
__global__ __launch_bounds__(256) void k_delta_prep(DeltaArgs a, DeltaRows r, int s, int n) {
  const int t = blockIdx.x, tid = threadIdx.x, l = tid & 15, grp = tid >> 4;
  const int DK = a.DK, C = a.C, taps = a.taps, KQ = a.KH * DK, VW = a.H * a.DV;
  const float *__restrict__ row = a.p + (int64_t)t * a.ldp;
  const int nb = min(taps - 1, n + t);
  // the raw row j steps back: of this portion, or of the history
  auto src = [&](int j) { return t >= j ? row - (int64_t)j * a.ldp : a.ring + (int64_t)((n + t - j) % taps) * C; };
  auto conv4 = [&](int ch) {
    float4 r4 = make_float4(0.f, 0.f, 0.f, 0.f);
    for (int j = 0; j <= nb; j++) {
      const float4 x = *(const float4 *)(src(j) + ch), w = *(const float4 *)(a.conv + (int64_t)j * C + ch);
      r4.x = fmaf(x.x, w.x, r4.x), r4.y = fmaf(x.y, w.y, r4.y), r4.z = fmaf(x.z, w.z, r4.z), r4.w = fmaf(x.w, w.w, r4.w);
    }
    return make_float4(delta_silu(r4.x), delta_silu(r4.y), delta_silu(r4.z), delta_silu(r4.w));
  };
  for (int item = grp; item < 2 * a.KH; item += 16) {
    const bool key = item >= a.KH;
    const int kh = key ? item - a.KH : item;
    float4 x[NC];
    float xx = 0.0f;
#pragma unroll
    for (int i = 0; i < NC; i++) {
      const int e = 4 * (l + 16 * i);
      x[i] = e < DK ? conv4((key ? KQ : 0) + kh * DK + e) : make_float4(0.f, 0.f, 0.f, 0.f);
      xx += x[i].x * x[i].x + x[i].y * x[i].y + x[i].z * x[i].z + x[i].w * x[i].w;
    }
    const float sc = 1.0f / (sqrtf(row16_sum(xx) + 1e-6f) * (key ? 1.0f : sqrtf((float)a.dk)));
    float *dst = (key ? r.K : r.Q) + (int64_t)t * KQ + kh * DK;
#pragma unroll
    for (int i = 0; i < NC; i++) {
      const int e = 4 * (l + 16 * i);
      if (e < DK) *(float4 *)(dst + e) = make_float4(x[i].x * sc, x[i].y * sc, x[i].z * sc, x[i].w * sc);
    }
  }
  for (int e = 4 * tid; e < VW; e += 1024) *(float4 *)(r.V + (int64_t)t * VW + e) = conv4(2 * KQ + e);
  for (int h = tid; h < a.H; h += 256) {
    r.BT[(int64_t)t * a.H + h] = 1.0f / (1.0f + expf(-row[C + VW + h]));
    r.LG[(int64_t)t * a.H + h] = delta_log_decay(a.neg_a[h], row[C + VW + a.H + h] + a.dt_bias[h]);
  }
}

// the recurrence token by token: 16 lanes per value column, a workgroup holds 16 columns of a head
template <int NC>
__global__ __launch_bounds__(256) void k_delta_scan(DeltaArgs a, DeltaRows r, float *__restrict__ out, int s, int n) {
  const int l = threadIdx.x & 15, h = blockIdx.x, c = blockIdx.y * 16 + (threadIdx.x >> 4);
  const int DK = a.DK, kh = h / (a.H / a.KH), KQ = a.KH * DK, VW = a.H * a.DV;
  float *__restrict__ Sc = a.S + ((int64_t)h * a.DV + c) * DK;  // DV is a multiple of 16
  float4 st[NC];
#pragma unroll
  for (int i = 0; i < NC; i++) {
    const int e = 4 * (l + 16 * i);
    st[i] = (n > 0 && e < DK) ? *(const float4 *)(Sc + e) : make_float4(0.f, 0.f, 0.f, 0.f);
  }
  struct Row {
    float4 q[NC], k[NC];
    float v, lg, bt;
  };
  auto load = [&](int t, Row &w) {
    t = min(t, s - 1);
#pragma unroll
    for (int i = 0; i < NC; i++) {
      const int e = 4 * (l + 16 * i);
      const float4 zero = make_float4(0.f, 0.f, 0.f, 0.f);
      w.q[i] = e < DK ? *(const float4 *)(r.Q + (int64_t)t * KQ + kh * DK + e) : zero;
      w.k[i] = e < DK ? *(const float4 *)(r.K + (int64_t)t * KQ + kh * DK + e) : zero;
    }
    w.v = r.V[(int64_t)t * VW + h * a.DV + c];
    w.lg = r.LG[(int64_t)t * a.H + h];
    w.bt = r.BT[(int64_t)t * a.H + h];
  };
  auto step = [&](int t, const Row &w) {
    const float g = expf(w.lg);
    float dot = 0.0f;
#pragma unroll
    for (int i = 0; i < NC; i++) {
      st[i].x *= g, st[i].y *= g, st[i].z *= g, st[i].w *= g;
      dot = fmaf(st[i].x, w.k[i].x, fmaf(st[i].y, w.k[i].y, fmaf(st[i].z, w.k[i].z, fmaf(st[i].w, w.k[i].w, dot))));
    }
    const float u = w.bt * (w.v - row16_sum(dot));
    float o = 0.0f;
#pragma unroll
    for (int i = 0; i < NC; i++) {
      st[i].x = fmaf(w.k[i].x, u, st[i].x), st[i].y = fmaf(w.k[i].y, u, st[i].y);
      st[i].z = fmaf(w.k[i].z, u, st[i].z), st[i].w = fmaf(w.k[i].w, u, st[i].w);
      o = fmaf(st[i].x, w.q[i].x, fmaf(st[i].y, w.q[i].y, fmaf(st[i].z, w.q[i].z, fmaf(st[i].w, w.q[i].w, o))));
    }
    o = row16_sum(o);
    if (l == 0) out[(int64_t)t * VW + h * a.DV + c] = o;
  };
  Row r0, r1;
  load(0, r0);
  int t = 0;
  for (; t + 2 <= s; t += 2) {
    load(t + 1, r1);
    step(t, r0);
    load(t + 2, r0);
    step(t + 1, r1);
  }
  if (t < s) step(t, r0);
#pragma unroll
  for (int i = 0; i < NC; i++) {
    const int e = 4 * (l + 16 * i);
    if (e < DK) *(float4 *)(Sc + e) = st[i];
  }
}

// a wavefront per (token, head): out <- out / rms(out) * norm * silu(gate)
__global__ __launch_bounds__(256) void k_delta_finish(DeltaArgs a, float *__restrict__ out, int64_t items) {
  const int lane = threadIdx.x & 63;
  const int64_t item = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (item >= items) return;
  const int64_t t = item / a.H;
  const int h = (int)(item % a.H);
  float *o = out + (t * a.H + h) * a.DV;
  const float *g = a.p + t * a.ldp + a.C + h * a.DV;
  float ss = 0.0f;
  for (int c = lane; c < a.DV; c += 64) ss = fmaf(o[c], o[c], ss);
  const float rstd = 1.0f / sqrtf(wave_sum(ss) / (float)a.dv + a.eps);
  for (int c = lane; c < a.DV; c += 64) o[c] = o[c] * rstd * a.norm[c] * delta_silu(g[c]);
}

// the raw rows of the last min(taps, s) tokens into the history
__global__ __launch_bounds__(256) void k_delta_history(DeltaArgs a, int s, int n) {
  const int t = s - 1 - (int)blockIdx.y;
  const int c = 4 * (blockIdx.x * 256 + threadIdx.x);
  if (t < 0 || c >= a.C) return;
  *(float4 *)(a.ring + (int64_t)((n + t) % a.taps) * a.C + c) = *(const float4 *)(a.p + (int64_t)t * a.ldp + c);
}

static DeltaRows delta_rows(const DeltaArgs &a, int s, float *w) {
  DeltaRows r;
  r.Q = w, w += (size_t)s * a.KH * a.DK;
  r.K = w, w += (size_t)s * a.KH * a.DK;
  r.V = w, w += (size_t)s * a.H * a.DV;
  r.LG = w, w += (size_t)s * a.H;
  r.BT = w;
  return r;
}
size_t delta_scratch_floats(const DeltaArgs &a, int s) { return (size_t)s * (2 * (size_t)a.KH * a.DK + (size_t)a.H * a.DV + 2 * (size_t)a.H); }

int launch_delta_rows(const DeltaArgs &a, float *out, int s, int n, float *scratch) {
  if (s <= 0) return 0;
  hipStream_t st = state().stream;
  const DeltaRows r = delta_rows(a, s, scratch);
  const int nc = (a.DK + 63) / 64;
  if (nc > 4) return fail(CTHIP_E_UNSUPPORTED, "delta rule: key heads of %d (at most 256)", a.DK);
  const dim3 gs(a.H, a.DV / 16);
#define GO(N)                                                                              \
  hipLaunchKernelGGL((k_delta_prep<N>), dim3(s), dim3(256), 0, st, a, r, s, n);            \
  hipLaunchKernelGGL((k_delta_scan<N>), gs, dim3(256), 0, st, a, r, out, s, n)
  if (nc <= 1) { GO(1); }
  else if (nc <= 2) { GO(2); }
  else { GO(4); }
#undef GO
  CTHIP_LAUNCH_CHECK();
  const int64_t items = (int64_t)s * a.H;
  hipLaunchKernelGGL(k_delta_finish, dim3((unsigned)((items + 3) / 4)), dim3(256), 0, st, a, out, items);
  const int keep = s < a.taps ? s : a.taps;
  hipLaunchKernelGGL(k_delta_history, dim3((unsigned)((a.C / 4 + 255) / 256), (unsigned)keep), dim3(256), 0, st, a, s, n);
  CTHIP_LAUNCH_CHECK();
  return 0;
}

}  // namespace cthip
