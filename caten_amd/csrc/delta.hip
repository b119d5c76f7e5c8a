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

// One token per launch.  Nothing that is asked for from memory waits for anything else: the state, the projection row, and
// every slot of the history with every tap's weights (which slot is how old is known when the position arrives).
// SLOTS: the most taps the unrolled convolution holds; longer ones take their history row by row.
template <int NC, int CPG>
__global__ __launch_bounds__(1024) void k_delta_step(DeltaArgs a, float *__restrict__ out, const int *__restrict__ tokpos,
                                                     const int *__restrict__ ctrl) {
  constexpr int SLOTS = 4;
  extern __shared__ float lds[];
  const int DK = a.DK, DV = a.DV, C = a.C, taps = a.taps;
  float *cs = lds;                 // q: DK, k: DK, v: DV of this head, convolved
  float *os = lds + 2 * DK + DV;   // DV outputs
  float *red = os + DV;            // 16 partial sums
  const int tid = threadIdx.x, nthr = blockDim.x, l = tid & 15, grp = tid >> 4, ngrp = nthr >> 4;
  const int h = blockIdx.x, rep = a.H / a.KH, kh = h / rep;
  const int qo = kh * DK, ko = a.KH * DK + kh * DK, vo = 2 * a.KH * DK + h * DV, go = C + h * DV, bo = C + a.H * DV + h;
  const float *__restrict__ p = a.p;
  float *__restrict__ Sh = a.S + (int64_t)h * DV * DK;
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
  const int pos = tokpos[1];
  const int stop = ctrl ? ctrl[1] : 0;
  const float pb = p[bo], pa = p[bo + a.H], na = a.neg_a[h], dt = a.dt_bias[h];
  const int nch = 2 * DK + DV;
  auto channel = [&](int c) { return c < DK ? qo + c : c < 2 * DK ? ko + c - DK : vo + c - 2 * DK; };
  const int ch0 = channel(min(tid, nch - 1));
  float cur = p[ch0], hist[SLOTS], wt[SLOTS];
#pragma unroll
  for (int j = 0; j < SLOTS; j++) {
    hist[j] = a.ring[(int64_t)min(j, taps - 1) * C + ch0];
    wt[j] = a.conv[(int64_t)min(j, taps - 1) * C + ch0];
  }
  load_state(0);
  const float gate0 = p[go + min(tid, DV - 1)], norm0 = a.norm[min(tid, DV - 1)];
  const bool ended = stop != 0;
  const int slot = pos % taps, nb = min(taps - 1, pos);
  auto keep = [&](int c, int ch, float x) {  // the raw row into the history; a key head's by the first of its value heads
    if (!ended && (c >= 2 * DK || h % rep == 0)) a.ring[(int64_t)slot * C + ch] = x;
  };
  if (taps <= SLOTS) {
    float r = cur * wt[0];
#pragma unroll
    for (int j = 1; j < SLOTS; j++) {
      int sl = slot - j;
      sl = sl < 0 ? sl + taps : sl;
      const float x = sl == 0 ? hist[0] : sl == 1 ? hist[1] : sl == 2 ? hist[2] : hist[3];
      if (j <= nb) r = fmaf(x, wt[j], r);
    }
    if (tid < nch) {
      cs[tid] = delta_silu(r);
      keep(tid, ch0, cur);
    }
  }
  for (int c = taps <= SLOTS ? tid + nthr : tid; c < nch; c += nthr) {
    const int ch = channel(c);
    const float x = p[ch];
    float r = x * a.conv[ch];
    for (int j = 1; j <= nb; j++) {
      int sl = slot - j;
      sl = sl < 0 ? sl + taps : sl;
      r = fmaf(a.ring[(int64_t)sl * C + ch], a.conv[(int64_t)j * C + ch], r);
    }
    cs[c] = delta_silu(r);
    keep(c, ch, x);
  }
  __syncthreads();
  float4 q[NC], k[NC];
  float qq = 0.0f, kk = 0.0f;
#pragma unroll
  for (int i = 0; i < NC; i++) {
    const int e = 4 * (l + 16 * i);
    q[i] = k[i] = make_float4(0.f, 0.f, 0.f, 0.f);
    if (e < DK) {
      q[i] = *(const float4 *)(cs + e);
      k[i] = *(const float4 *)(cs + DK + e);
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
  const float beta = 1.0f / (1.0f + expf(-pb));
  const float g = expf(delta_log_decay(na, pa + dt));
  float o2 = 0.0f;
  for (int c0 = 0; c0 < DV; c0 += ngrp * CPG) {
    if (c0 > 0) load_state(c0);
#pragma unroll
    for (int kc = 0; kc < CPG; kc++) {
      const int c = c0 + grp + ngrp * kc;
      const bool in = c < DV;
      const float v = cs[2 * DK + (in ? c : 0)];
      float dot = 0.0f;
#pragma unroll
      for (int i = 0; i < NC; i++) {
        float4 &t = s[kc][i];
        if (pos == 0) t = make_float4(0.f, 0.f, 0.f, 0.f);  // a sequence starts from zero, whatever the one before it left
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
      }
    }
  }
  o2 = wave_sum(o2);
  if ((tid & 63) == 0) red[tid >> 6] = o2;
  __syncthreads();
  float sum = 0.0f;
  for (int w = 0; w < (nthr >> 6); w++) sum += red[w];
  const float rstd = 1.0f / sqrtf(sum / (float)a.dv + a.eps);
  for (int c = tid; c < DV; c += nthr)
    out[(int64_t)h * DV + c] = os[c] * rstd * (c == tid ? norm0 : a.norm[c]) * delta_silu(c == tid ? gate0 : p[go + c]);
}

int launch_delta_step(const DeltaArgs &a, float *out, const int *tokpos, const int *ctrl) {
  // 16 lanes per value column, whole wavefronts
  int block = 16 * a.DV;
  if (block > 1024) block = 1024;
  const size_t lds = sizeof(float) * (size_t)(2 * a.DK + 2 * a.DV + 16);
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

// ---- the recurrence chunk by chunk ----
// Over a chunk of 64 tokens, with G_i the sum of the logarithms of the decays up to token i and S the state before it,
//   u_i = beta_i (v_i - e^{G_i} S^T k_i - sum_{j<i} e^{G_i - G_j} (k_i . k_j) u_j),
// so with A_ij = beta_i e^{G_i - G_j} k_i . k_j (j < i):  (I + A) U = diag(beta) V - diag(beta e^G) K S.  Hence
//   [W | U0] = (I + A)^-1 [diag(beta e^G) K | diag(beta) V]   k_delta_chunk: every chunk and head by itself;
//   U = U0 - W S,  O = diag(e^G) Q S + P U,  S <- e^{G_63} S + K^T diag(e^{G_63 - G}) U,   P_ij = e^{G_i - G_j} q_i . k_j (j <= i)
//                                                           k_delta_apply: the chunks in order, 16 value columns a workgroup.
// Everything is fp32 (v_mfma_f32_16x16x4_f32); the sums G are kept in double precision, since strong decays make them large
// while the differences that count stay small.
//
// Operand order: lane l supplies a row's four floats 4 (l/16) .. of a 16-float piece to four matrix instructions, and a result
// tile holds rows 4 (l/16) + i of column l % 16 in register i -- so a result tile is the right-hand operand of a further
// product as it is, piece = tile, instruction = register.
constexpr int kChunk = 64;
constexpr int kChunkFrom = 32;  // shorter portions go token by token
typedef float v4f_t __attribute__((ext_vector_type(4)));
struct DeltaChunks {
  float *W, *U, *P, *E1, *E2;  // per (chunk, head): [64][DK], [64][DV], [64][64] (lower tiles), e^{G_i}, e^{G_63 - G_i}
};

__device__ __forceinline__ v4f_t mfma4(const float4 a, const v4f_t b, v4f_t c) {
  c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.x, b[0], c, 0, 0, 0);
  c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.y, b[1], c, 0, 0, 0);
  c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.z, b[2], c, 0, 0, 0);
  return __builtin_amdgcn_mfma_f32_16x16x4f32(a.w, b[3], c, 0, 0, 0);
}

__global__ __launch_bounds__(256) void k_delta_chunk(DeltaArgs a, DeltaRows r, DeltaChunks w, int s) {
  constexpr int LA = kChunk + 4;
  __shared__ __align__(16) float Am[kChunk][LA];
  __shared__ __align__(16) float Tb[4][16][20];
  __shared__ double Gs[kChunk];
  __shared__ float Bs[kChunk];
  const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6, lo = lane & 15, hi = lane >> 4;
  const int c0 = blockIdx.x * kChunk, h = blockIdx.y, kh = h / (a.H / a.KH);
  const int DK = a.DK, DV = a.DV, KQ = a.KH * DK, VW = a.H * DV;
  const int64_t item = (int64_t)blockIdx.x * a.H + h;
  const float *__restrict__ Kr = r.K + kh * DK, *__restrict__ Qr = r.Q + kh * DK, *__restrict__ Vr = r.V + h * DV;
  auto tok = [&](int i) { return (int64_t)min(c0 + i, s - 1); };  // rows past the end repeat the last one; their steps are zero
  if (wv == 0) {
    const bool in = c0 + lane < s;
    double g = in ? (double)r.LG[tok(lane) * a.H + h] : 0.0;
#pragma unroll
    for (int d = 1; d < 64; d <<= 1) {
      const double t = __shfl_up(g, d, 64);
      if (lane >= d) g += t;
    }
    Gs[lane] = g;
    Bs[lane] = in ? r.BT[tok(lane) * a.H + h] : 0.0f;
    const double gl = __shfl(g, 63, 64);
    w.E1[item * kChunk + lane] = expf((float)g);
    w.E2[item * kChunk + lane] = expf((float)(gl - g));
  }
  __syncthreads();
  // ten lower tiles of K K^T and of Q K^T, dealt to the wavefronts
  float *__restrict__ P = w.P + item * kChunk * kChunk;
  for (int it = wv; it < 20; it += 4) {
    const bool qk = it >= 10;
    int rest = qk ? it - 10 : it, ti = 0;
    while (rest > ti) rest -= ++ti;
    const int tj = rest;
    const float *ar = (qk ? Qr : Kr) + tok(16 * ti + lo) * KQ + 4 * hi;
    const float *br = Kr + tok(16 * tj + lo) * KQ + 4 * hi;
    v4f_t acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 8
    for (int c = 0; c < DK; c += 16) {
      const float4 bv = *(const float4 *)(br + c);
      acc = mfma4(*(const float4 *)(ar + c), v4f_t{bv.x, bv.y, bv.z, bv.w}, acc);
    }
    const int j = 16 * tj + lo;
#pragma unroll
    for (int t = 0; t < 4; t++) {
      const int i = 16 * ti + 4 * hi + t;
      const float e = expf((float)(Gs[i] - Gs[j])) * acc[t];
      if (qk) P[i * kChunk + j] = j <= i ? e : 0.0f;
      else Am[i][j] = j < i ? Bs[i] * e : 0.0f;
    }
  }
  __syncthreads();
  if (wv == 0) {  // inverses of the four diagonal tiles of I + A: lane = column lo of tile hi
    float x[16];
#pragma unroll
    for (int i = 0; i < 16; i++) {
      float t = i == lo ? 1.0f : 0.0f;
#pragma unroll
      for (int m = 0; m < i; m++) t = fmaf(-Am[16 * hi + i][16 * hi + m], x[m], t);
      x[i] = t;
      Tb[hi][i][lo] = t;
    }
  }
  __syncthreads();
  // forward substitution over the four row tiles, every 16 columns of [K | V] by themselves
  for (int ct = wv; ct < (DK + DV) / 16; ct += 4) {
    const bool key = 16 * ct < DK;
    const int e = key ? 16 * ct + lo : 16 * ct - DK + lo;
    float b[4][4];
#pragma unroll
    for (int bt = 0; bt < 4; bt++)
#pragma unroll
      for (int t = 0; t < 4; t++) {
        const int64_t tk = tok(16 * bt + 4 * hi + t);
        b[bt][t] = key ? Kr[tk * KQ + e] : Vr[tk * VW + e];
      }
    v4f_t X[4];
#pragma unroll
    for (int bt = 0; bt < 4; bt++) {
      v4f_t acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int c = 0; c < bt; c++) acc = mfma4(*(const float4 *)&Am[16 * bt + lo][16 * c + 4 * hi], X[c], acc);
#pragma unroll
      for (int t = 0; t < 4; t++) {
        const int i = 16 * bt + 4 * hi + t;
        acc[t] = b[bt][t] * (key ? Bs[i] * expf((float)Gs[i]) : Bs[i]) - acc[t];
      }
      X[bt] = mfma4(*(const float4 *)&Tb[bt][lo][4 * hi], acc, v4f_t{0.f, 0.f, 0.f, 0.f});
    }
    float *dst = key ? w.W + item * kChunk * DK + e : w.U + item * kChunk * DV + e;
    const int ld = key ? DK : DV;
#pragma unroll
    for (int bt = 0; bt < 4; bt++)
#pragma unroll
      for (int t = 0; t < 4; t++) dst[(int64_t)(16 * bt + 4 * hi + t) * ld] = X[bt][t];
  }
}

// NK: 16-key tiles of the state a workgroup holds (DK <= 16 NK); wavefront w owns row tile w of the chunk and the state's tiles
// w, w + 4, ...; every wavefront holds the whole 16-column state as a right-hand operand.  The next chunk's operands are
// requested as soon as this chunk's have been multiplied.
template <int NK>
__global__ __launch_bounds__(256) void k_delta_apply(DeltaArgs a, DeltaRows r, DeltaChunks w, float *__restrict__ out, int s, int n) {
  __shared__ v4f_t Us[4][64], Ss[NK][64];
  const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6, lo = lane & 15, hi = lane >> 4;
  const int h = blockIdx.x, col = blockIdx.y * 16 + lo, kh = h / (a.H / a.KH);
  const int DK = a.DK, DV = a.DV, KQ = a.KH * DK, VW = a.H * DV, nk = DK >> 4, nch = (s + kChunk - 1) / kChunk;
  const float *__restrict__ Kr = r.K + kh * DK, *__restrict__ Qr = r.Q + kh * DK;
  float *__restrict__ Sc = a.S + ((int64_t)h * DV + col) * DK + 4 * hi;
  const v4f_t zero = {0.f, 0.f, 0.f, 0.f};
  v4f_t S[NK], own[NK / 4];
  auto state_tile = [&](int mt) {
    if (n == 0 || mt >= nk) return zero;
    return *(const v4f_t *)(Sc + 16 * mt);
  };
#pragma unroll
  for (int c = 0; c < NK; c++) S[c] = state_tile(c);
#pragma unroll
  for (int k = 0; k < NK / 4; k++) own[k] = state_tile(wv + 4 * k);
  auto tok = [&](int ch, int i) { return (int64_t)min(ch * kChunk + i, s - 1); };
  float4 Wr[NK], Qa[NK], Pr[4], e2[4];
  float Kt[NK / 4][16], u0[4];
  float4 e1;
  float gl;
  auto load_wq = [&](int ch) {
    const float *wr = w.W + (((int64_t)ch * a.H + h) * kChunk + 16 * wv + lo) * DK + 4 * hi;
    const float *qr = Qr + tok(ch, 16 * wv + lo) * KQ + 4 * hi;
#pragma unroll
    for (int c = 0; c < NK; c++) {
      const int e = 16 * min(c, nk - 1);  // (past the end: times zero state)
      Wr[c] = *(const float4 *)(wr + e);
      Qa[c] = *(const float4 *)(qr + e);
    }
    const float *ur = w.U + (((int64_t)ch * a.H + h) * kChunk + 16 * wv + 4 * hi) * DV + col;
#pragma unroll
    for (int i = 0; i < 4; i++) u0[i] = ur[(int64_t)i * DV];
    e1 = *(const float4 *)(w.E1 + ((int64_t)ch * a.H + h) * kChunk + 16 * wv + 4 * hi);
  };
  auto load_p = [&](int ch) {
    const float *pr = w.P + (((int64_t)ch * a.H + h) * kChunk + 16 * wv + lo) * kChunk + 4 * hi;
#pragma unroll
    for (int c = 0; c < 4; c++) Pr[c] = *(const float4 *)(pr + 16 * min(c, wv));  // (tiles above the diagonal are not used)
  };
  auto load_k = [&](int ch) {
#pragma unroll
    for (int k = 0; k < NK / 4; k++) {
      const int e = 16 * min(wv + 4 * k, nk - 1) + lo;
#pragma unroll
      for (int c = 0; c < 4; c++)
#pragma unroll
        for (int t = 0; t < 4; t++) Kt[k][4 * c + t] = Kr[tok(ch, 16 * c + 4 * hi + t) * KQ + e];
    }
    const float *er = w.E2 + ((int64_t)ch * a.H + h) * kChunk + 4 * hi;
#pragma unroll
    for (int c = 0; c < 4; c++) e2[c] = *(const float4 *)(er + 16 * c);
    gl = w.E1[((int64_t)ch * a.H + h) * kChunk + kChunk - 1];
  };
  load_wq(0);
  load_p(0);
  load_k(0);
  for (int ch = 0; ch < nch; ch++) {
    const int nx = min(ch + 1, nch - 1);
    v4f_t u = zero, o = zero;
#pragma unroll
    for (int c = 0; c < NK; c++) {
      u = mfma4(Wr[c], S[c], u);
      o = mfma4(Qa[c], S[c], o);
    }
#pragma unroll
    for (int i = 0; i < 4; i++) u[i] = u0[i] - u[i];
    o[0] *= e1.x, o[1] *= e1.y, o[2] *= e1.z, o[3] *= e1.w;
    Us[wv][lane] = u;
    load_wq(nx);
    __syncthreads();
    v4f_t U[4];
#pragma unroll
    for (int c = 0; c < 4; c++) {
      U[c] = Us[c][lane];
      if (c <= wv) o = mfma4(Pr[c], U[c], o);
    }
    load_p(nx);
#pragma unroll
    for (int i = 0; i < 4; i++) {
      const int t = ch * kChunk + 16 * wv + 4 * hi + i;
      if (t < s) out[(int64_t)t * VW + h * DV + col] = o[i];
    }
#pragma unroll
    for (int c = 0; c < 4; c++) U[c][0] *= e2[c].x, U[c][1] *= e2[c].y, U[c][2] *= e2[c].z, U[c][3] *= e2[c].w;
#pragma unroll
    for (int k = 0; k < NK / 4; k++) {
      own[k] *= gl;
#pragma unroll
      for (int c = 0; c < 4; c++)
#pragma unroll
        for (int t = 0; t < 4; t++) own[k] = __builtin_amdgcn_mfma_f32_16x16x4f32(Kt[k][4 * c + t], U[c][t], own[k], 0, 0, 0);
      Ss[wv + 4 * k][lane] = own[k];
    }
    load_k(nx);
    __syncthreads();
#pragma unroll
    for (int c = 0; c < NK; c++) S[c] = c < nk ? Ss[c][lane] : zero;
  }
#pragma unroll
  for (int k = 0; k < NK / 4; k++)
    if (wv + 4 * k < nk) *(v4f_t *)(Sc + 16 * (wv + 4 * k)) = own[k];
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
static size_t delta_rows_floats(const DeltaArgs &a, int s) {
  return ((size_t)s * (2 * (size_t)a.KH * a.DK + (size_t)a.H * a.DV + 2 * (size_t)a.H) + 3) & ~(size_t)3;
}
size_t delta_scratch_floats(const DeltaArgs &a, int s) {
  const size_t chunks = s < kChunkFrom ? 0 : (s + kChunk - 1) / kChunk;
  return delta_rows_floats(a, s) + chunks * a.H * kChunk * (size_t)(a.DK + a.DV + kChunk + 2);
}

int launch_delta_rows(const DeltaArgs &a, float *out, int s, int n, float *scratch) {
  if (s <= 0) return 0;
  hipStream_t st = state().stream;
  const DeltaRows r = delta_rows(a, s, scratch);
  const int nc = (a.DK + 63) / 64;
  if (nc > 4) return fail(CTHIP_E_UNSUPPORTED, "delta rule: key heads of %d (at most 256)", a.DK);
  const dim3 gs(a.H, a.DV / 16), b256(256);
#define GO(N)                                                                    \
  hipLaunchKernelGGL((k_delta_prep<N>), dim3(s), b256, 0, st, a, r, s, n);       \
  if (s < kChunkFrom) hipLaunchKernelGGL((k_delta_scan<N>), gs, b256, 0, st, a, r, out, s, n)
  if (nc <= 1) { GO(1); }
  else if (nc <= 2) { GO(2); }
  else { GO(4); }
  CTHIP_LAUNCH_CHECK();
  if (s >= kChunkFrom) {
    const size_t chunks = (s + kChunk - 1) / kChunk, rows = chunks * a.H * kChunk;
    DeltaChunks w;
    w.W = scratch + delta_rows_floats(a, s);
    w.U = w.W + rows * a.DK;
    w.P = w.U + rows * a.DV;
    w.E1 = w.P + rows * kChunk;
    w.E2 = w.E1 + rows;
    hipLaunchKernelGGL(k_delta_chunk, dim3((unsigned)chunks, (unsigned)a.H), b256, 0, st, a, r, w, s);
    if (nc <= 1) hipLaunchKernelGGL((k_delta_apply<4>), gs, b256, 0, st, a, r, w, out, s, n);
    else if (nc <= 2) hipLaunchKernelGGL((k_delta_apply<8>), gs, b256, 0, st, a, r, w, out, s, n);
    else hipLaunchKernelGGL((k_delta_apply<16>), gs, b256, 0, st, a, r, w, out, s, n);
  }
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
