// A decode step of a layer whose mixers are attention over a sliding window (window.hip), lightning attention
// (lightning.hip), or the two side by side: one launch, whose workgroups belong to one mixer or the other.
//
//   window     workgroup (key range, key/value head, up to QB of its query heads).  It takes the root mean squares of all
//              queries and keys, normalises and rotates its own, and attends over its share of the ring: 16 lanes per row,
//              16 rows a tile, range r takes the r-th run of `2^lper` tiles.  Rings are walked by row, not by position; which
//              position a row holds follows from the step's.  The new key and value come from the projection row; the range
//              that owns their row of the ring stores them.  While
//              few rows are held, few ranges have any, and a single one finishes by itself.  Every group of 16 lanes keeps a
//              softmax of its own; they meet in LDS.
//   lightning  workgroup (head, 16 value columns), 16 lanes per column: the state's rows are read once, updated, read out
//              and written once.  The norm takes all heads' outputs.
//
// What meets across workgroups -- a head's key ranges, the heads' outputs in front of the norm -- is left in memory with
// device-scope stores, a ticket is drawn, and the workgroup with the last ticket finishes (as k_attn_cached does).
#include <type_traits>

#include "common.h"
#include "mixers.h"

namespace cthip {

constexpr int kWindowTiles = 4;  // tiles of a key range, at least
struct WindowShape {
  int ranges, lper;  // key ranges of 2^lper tiles each
  int rep, qgroups;  // query heads per key/value head; workgroups of up to QB of them
  unsigned inv;      // about 2^32 / rows
  int blocks() const { return ranges * heads; }
  int heads;         // workgroups of a range
};
static int window_pieces(const WindowArgs &a) { return ((a.DK > a.DV ? a.DK : a.DV) + 63) / 64; }
static int window_qb(const WindowArgs &a) {  // (heads past 128 entries: what two of them keep fits LDS)
  const int rep = a.H / a.G;
  return rep >= 3 && window_pieces(a) <= 2 ? 4 : rep >= 2 ? 2 : 1;
}
static WindowShape window_shape(const WindowArgs &a) {
  WindowShape w;
  w.rep = a.H / a.G;
  w.qgroups = (w.rep + window_qb(a) - 1) / window_qb(a);
  w.heads = a.G * w.qgroups;
  const int tiles = (a.rows + 15) / 16, fill = 512 / w.heads;
  const int most = fill < 1 ? 1 : fill < kWindowMaxRanges ? fill : kWindowMaxRanges;
  for (w.lper = 0; (1 << w.lper) < kWindowTiles || ((tiles - 1) >> w.lper) + 1 > most; w.lper++) {}
  w.ranges = ((tiles - 1) >> w.lper) + 1;
  w.inv = a.rows > 1 ? (unsigned)((1ull << 32) / (unsigned)a.rows) : 0xffffffffu;
  return w;
}
constexpr int part_pitch(int dv) { return dv + 4; }  // a range's record of one head: DV sums, maximum, denominator, two unused
int window_tickets(const WindowArgs &a) { return window_shape(a).heads; }
size_t window_part_floats(const WindowArgs &a) { return (size_t)window_shape(a).blocks() * window_qb(a) * part_pitch(a.DV); }
size_t lightning_raw_floats(const LightningArgs &a) { return (size_t)a.H * a.DV; }

__device__ __forceinline__ float agent_load(const float *p) { return __hip_atomic_load(p, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT); }
__device__ __forceinline__ void agent_store(float *p, float v) { __hip_atomic_store(p, v, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT); }
// two floats at an address that is a multiple of 8
__device__ __forceinline__ float2 agent_load2(const float *p) {
  return __builtin_bit_cast(float2, __hip_atomic_load((const unsigned long long *)p, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT));
}
__device__ __forceinline__ void agent_store2(float *p, float2 v) {
  __hip_atomic_store((unsigned long long *)p, __builtin_bit_cast(unsigned long long, v), __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
}

// true in the workgroup that draws the last of `n` tickets; every thread's stores have reached memory by then
__device__ __forceinline__ bool last_ticket(int *count, int n, int *lds) {
  asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
  __syncthreads();
  if (threadIdx.x == 0) *lds = __hip_atomic_fetch_add(count, 1, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
  __syncthreads();
  if (*lds != n - 1) return false;
  if (threadIdx.x == 0) __hip_atomic_store(count, 0, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);  // the next launch counts again
  return true;
}

template <int NC, int QB>
struct StepLds {
  float q[QB][64 * NC], k[64 * NC];
  float o[16][QB][64 * NC], m[16][QB], l[16][QB];  // of every group of 16 lanes
  float red[8];
  int ticket;
};

// NC: 64-entry pieces of a head, at most; QB: query heads of a workgroup
template <int NC, int QB>
__device__ void window_step(const WindowArgs &a, const WindowShape &sh, int hg, int range, float *__restrict__ part, int *__restrict__ count,
                            float *__restrict__ out, const int *__restrict__ tokpos, StepLds<NC, QB> &S) {
  constexpr int U = NC >= 4 ? 2 : 4;  // tiles a wavefront works on together
  constexpr int DP = 64 * NC, QE = (QB * DP + 255) / 256, SB = 4;
  const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6, g16 = lane >> 4, l = lane & 15;
  const int rep = sh.rep, g = sh.qgroups == 1 ? hg : hg / sh.qgroups, qg = hg - g * sh.qgroups;
  const int h0 = g * rep + qg * QB, nq = min(QB, (g + 1) * rep - h0);  // this workgroup's query heads
  const int DK = a.DK, DV = a.DV, KW = a.G * DK, VW = a.G * DV, QW = a.H * DK, rows = a.rows, half = a.rope ? a.half : 0;
  const float *__restrict__ pq = a.p, *__restrict__ pk = pq + QW, *__restrict__ pv = pk + KW;
  const int pos = tokpos[1];
  // ---- this step's queries, key and value ----
  auto mate = [&](int d) { return d < half ? d + half : d < 2 * half ? d - half : d; };
  auto square = [](const float4 x, float s) { return fmaf(x.x, x.x, fmaf(x.y, x.y, fmaf(x.z, x.z, fmaf(x.w, x.w, s)))); };
  float4 x[SB], y;
  if (a.qnorm) {
#pragma unroll
    for (int b = 0; b < SB; b++) x[b] = *(const float4 *)(pq + min(4 * tid + 1024 * b, QW - 4));
    y = *(const float4 *)(pk + min(4 * tid, KW - 4));
  }
  float qa[QE], qb[QE], wa[QE], wb[QE];
#pragma unroll
  for (int j = 0; j < QE; j++) {
    const int it = tid + 256 * j, h = min(it / DP, nq - 1), d = min(it % DP, DK - 1);
    const int e = (h0 + h) * DK + d, f = (h0 + h) * DK + mate(d);
    qa[j] = pq[e], qb[j] = pq[f];
    wa[j] = a.qnorm ? a.qnorm[e] : 1.0f, wb[j] = a.qnorm ? a.qnorm[f] : 1.0f;
  }
  const int kd = min(tid, DK - 1);
  const float ka = pk[g * DK + kd], kb = pk[g * DK + mate(kd)];
  const float wka = a.knorm ? a.knorm[g * DK + kd] : 1.0f, wkb = a.knorm ? a.knorm[g * DK + mate(kd)] : 1.0f;
  float4 vn[NC];
#pragma unroll
  for (int i = 0; i < NC; i++) vn[i] = *(const float4 *)(pv + g * DV + min(4 * (l + 16 * i), DV - 4));
  // ---- rows of the ring ----
  float4 kr[U][NC], vr[U][NC];
  auto request = [&](int u, int tile) {
    const int64_t row = min(tile * 16 + 4 * wv + g16, rows - 1);
#pragma unroll
    for (int i = 0; i < NC; i++) {
      kr[u][i] = *(const float4 *)(a.K + row * KW + g * DK + min(4 * (l + 16 * i), DK - 4));  // (past the head: times zero)
      vr[u][i] = *(const float4 *)(a.V + row * VW + g * DV + min(4 * (l + 16 * i), DV - 4));  // (past the head: not stored)
    }
  };
  const int first = range << sh.lper;
  const int held = min(pos + 1, rows), tiles = (held + 15) >> 4, nr = ((tiles - 1) >> sh.lper) + 1;
  if (range >= nr) return;  // no row of this range yet (uniform)
  const int end = min(first + (1 << sh.lper), tiles);
#pragma unroll
  for (int u = 0; u < U; u++) request(u, first + u);
  float qs = 1.0f, ks = 1.0f;
  if (a.qnorm) {
    float sq = 0.0f, sk = 4 * tid < KW ? square(y, 0.0f) : 0.0f;
#pragma unroll
    for (int b = 0; b < SB; b++)
      if (4 * tid + 1024 * b < QW) sq = square(x[b], sq);
    for (int e = 4 * tid + 1024 * SB; e < QW; e += 1024) sq = square(*(const float4 *)(pq + e), sq);
    for (int e = 4 * tid + 1024; e < KW; e += 1024) sk = square(*(const float4 *)(pk + e), sk);
    sq = wave_sum(sq), sk = wave_sum(sk);
    if (lane == 0) S.red[wv] = sq, S.red[4 + wv] = sk;
  }
  float2 qc[QE], kc = make_float2(1.0f, 0.0f);
  auto angle = [&](int d) { return d < 2 * half ? a.rope[(int64_t)pos * half + (d < half ? d : d - half)] : make_float2(1.0f, 0.0f); };
#pragma unroll
  for (int j = 0; j < QE; j++) qc[j] = angle(min((tid + 256 * j) % DP, DK - 1));
  kc = angle(kd);
  __syncthreads();
  if (a.qnorm) {
    qs = 1.0f / sqrtf(((S.red[0] + S.red[1]) + (S.red[2] + S.red[3])) / (float)(a.H * a.dk) + a.eps);
    ks = 1.0f / sqrtf(((S.red[4] + S.red[5]) + (S.red[6] + S.red[7])) / (float)(a.G * a.dk) + a.eps);
  }
  // entry d of a pair with its mate: the first is u cos - v sin, the second v cos + u sin
  auto turned = [&](int d, float x, float y, float2 c) {
    if (d >= 2 * half) return x;
    float o0, o1;
    if (d < half) rope_pair(x, y, c.y, c.x, o0, o1);
    else rope_pair(y, x, c.y, c.x, o0, o1);
    return d < half ? o0 : o1;
  };
#pragma unroll
  for (int j = 0; j < QE; j++) {  // (zero past the head and past the last query head)
    const int it = tid + 256 * j, h = it / DP, d = it % DP;
    if (h < QB) S.q[h][d] = h < nq && d < DK ? turned(d, qa[j] * qs * wa[j], qb[j] * qs * wb[j], qc[j]) * a.scale : 0.0f;
  }
  if (tid < DP) S.k[tid] = tid < DK ? turned(tid, ka * ks * wka, kb * ks * wkb, kc) : 0.0f;
  __syncthreads();
  int cur = pos - (int)__umulhi((unsigned)pos, sh.inv) * rows;  // pos mod rows
  while (cur >= rows) cur -= rows;
  float4 q[QB][NC], o[QB][NC], kn[NC];
  float m[QB], L[QB];
#pragma unroll
  for (int i = 0; i < NC; i++) {
    const int e = 4 * (l + 16 * i);
    kn[i] = *(const float4 *)&S.k[e];
#pragma unroll
    for (int h = 0; h < QB; h++) q[h][i] = *(const float4 *)&S.q[h][e], o[h][i] = make_float4(0.f, 0.f, 0.f, 0.f);
  }
#pragma unroll
  for (int h = 0; h < QB; h++) m[h] = -INFINITY, L[h] = 0.0f;
  if (cur >> (4 + sh.lper) == range && qg == 0 && tid < 16) {  // the new row: nobody reads this row of the ring in this step
#pragma unroll
    for (int i = 0; i < NC; i++) {
      const int e = 4 * (l + 16 * i);
      if (e < DK) *(float4 *)(a.K + (int64_t)cur * KW + g * DK + e) = kn[i];
      if (e < DV) *(float4 *)(a.V + (int64_t)cur * VW + g * DV + e) = vn[i];
    }
  }
  for (int tile0 = first; tile0 < end; tile0 += U) {
    if (tile0 != first) {
#pragma unroll
      for (int u = 0; u < U; u++) request(u, tile0 + u);
    }
    bool ok[U];
#pragma unroll
    for (int u = 0; u < U; u++) {
      const int slot = (tile0 + u) * 16 + 4 * wv + g16;
      int back = cur - slot;
      back += back < 0 ? rows : 0;
      ok[u] = tile0 + u < end && slot < rows && back <= pos && back < a.window;
      if (slot == cur) {
#pragma unroll
        for (int i = 0; i < NC; i++) kr[u][i] = kn[i], vr[u][i] = vn[i];
      }
      if (!ok[u]) {  // rows that no token of this sequence has written need not hold numbers
#pragma unroll
        for (int i = 0; i < NC; i++) vr[u][i] = make_float4(0.f, 0.f, 0.f, 0.f);
      }
    }
#pragma unroll
    for (int h = 0; h < QB; h++) {
      float sc[U], m_new = m[h];
#pragma unroll
      for (int u = 0; u < U; u++) {
        float d = 0.0f;
#pragma unroll
        for (int i = 0; i < NC; i++)
          d = fmaf(q[h][i].x, kr[u][i].x, fmaf(q[h][i].y, kr[u][i].y, fmaf(q[h][i].z, kr[u][i].z, fmaf(q[h][i].w, kr[u][i].w, d))));
        d = row16_sum(d);
        sc[u] = ok[u] ? d : -INFINITY;
        m_new = fmaxf(m_new, sc[u]);
      }
      const float m_use = m_new == -INFINITY ? 0.0f : m_new;  // no row of this group's yet
      const float corr = ct_exp(m[h] - m_use);
      float pr[U];
      L[h] *= corr;
#pragma unroll
      for (int u = 0; u < U; u++) {
        pr[u] = ct_exp(sc[u] - m_use);
        L[h] += pr[u];
      }
      m[h] = m_new;
#pragma unroll
      for (int i = 0; i < NC; i++) {
        float4 t = o[h][i];
        t.x *= corr, t.y *= corr, t.z *= corr, t.w *= corr;
#pragma unroll
        for (int u = 0; u < U; u++)
          t.x = fmaf(pr[u], vr[u][i].x, t.x), t.y = fmaf(pr[u], vr[u][i].y, t.y), t.z = fmaf(pr[u], vr[u][i].z, t.z), t.w = fmaf(pr[u], vr[u][i].w, t.w);
        o[h][i] = t;
      }
    }
  }
  const int group = 4 * wv + g16;
#pragma unroll
  for (int h = 0; h < QB; h++) {
#pragma unroll
    for (int i = 0; i < NC; i++) *(float4 *)&S.o[group][h][4 * (l + 16 * i)] = o[h][i];
    if (l == 0) S.m[group][h] = m[h], S.l[group][h] = L[h];
  }
  __syncthreads();
  const int og = QW + KW + VW;  // the gate in the projection row
  auto put = [&](int h, int c, float2 v, float den) {
    const int e = (h0 + h) * DV + c;
    const float f = a.out_scale / den;
    float2 y = make_float2(v.x * f, v.y * f);
    if (a.gated) {
      const float2 z = *(const float2 *)(a.p + og + e);
      y.x *= ct_sigmoid(z.x), y.y *= ct_sigmoid(z.y);
    }
    *(float2 *)(out + e) = y;
  };
  for (int it = tid; it < QB * DP / 2; it += 256) {
    const int h = it / (DP / 2), c = 2 * (it % (DP / 2));
    if (h >= nq || c >= DV) continue;
    float M = S.m[0][h];
#pragma unroll
    for (int w = 1; w < 16; w++) M = fmaxf(M, S.m[w][h]);
    const float Mu = M == -INFINITY ? 0.0f : M;
    float2 v = make_float2(0.f, 0.f);
    float den = 0.0f;
#pragma unroll
    for (int w = 0; w < 16; w++) {
      const float e = ct_exp(S.m[w][h] - Mu);
      const float2 t = *(const float2 *)&S.o[w][h][c];
      v.x = fmaf(e, t.x, v.x), v.y = fmaf(e, t.y, v.y);
      den = fmaf(e, S.l[w][h], den);
    }
    if (nr == 1) {
      if (a.sink) {
        const float sk = a.sink[h0 + h], top = fmaxf(M, sk), cr = ct_exp(M - top);
        v.x *= cr, v.y *= cr;
        den = fmaf(den, cr, ct_exp(sk - top));
      }
      put(h, c, v, den);
    } else {
      float *rec = part + ((int64_t)(hg * sh.ranges + range) * QB + h) * part_pitch(DV);
      agent_store2(rec + c, v);
      if (c == 0) agent_store2(rec + DV, make_float2(M, den));
    }
  }
  if (nr == 1) return;
  if (!last_ticket(count + hg, nr, &S.ticket)) return;
  auto merge = [&](auto width) {  // up to N records, all of them requested before the first is used
    constexpr int N = decltype(width)::value;
    for (int it = tid; it < QB * DP / 2; it += 256) {
      const int h = it / (DP / 2), c = 2 * (it % (DP / 2));
      if (h >= nq || c >= DV) continue;
      const float *rec = part + ((int64_t)hg * sh.ranges * QB + h) * part_pitch(DV);
      const int64_t pitch = (int64_t)QB * part_pitch(DV);
      float2 ml[N], ov[N];
#pragma unroll
      for (int r = 0; r < N; r++) {
        const float *t = rec + min(r, nr - 1) * pitch;
        ml[r] = agent_load2(t + DV), ov[r] = agent_load2(t + c);
      }
      float M = a.sink ? a.sink[h0 + h] : -INFINITY;
#pragma unroll
      for (int r = 0; r < N; r++) M = fmaxf(M, ml[r].x);  // (the last one again and again)
      float2 v = make_float2(0.f, 0.f);
      float den = a.sink ? ct_exp(a.sink[h0 + h] - M) : 0.0f;
#pragma unroll
      for (int r = 0; r < N; r++)
        if (r < nr) {
          const float e = ct_exp(ml[r].x - M);
          v.x = fmaf(e, ov[r].x, v.x), v.y = fmaf(e, ov[r].y, v.y);
          den = fmaf(e, ml[r].y, den);
        }
      put(h, c, v, den);
    }
  };
  if (nr <= 4) merge(std::integral_constant<int, 4>{});
  else if (nr <= 16) merge(std::integral_constant<int, 16>{});
  else merge(std::integral_constant<int, kWindowMaxRanges>{});
}

template <int NC>
__device__ void lightning_step(const LightningArgs &a, int block, int nblocks, float *__restrict__ raw, int *__restrict__ count,
                               float *__restrict__ out, const int *__restrict__ tokpos, const int *__restrict__ ctrl, float *red, int *ticket) {
  const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6, l = tid & 15, grp = tid >> 4;
  const int DK = a.DK, DV = a.DV, per = DV >> 4, h = block / per, c = (block - h * per) * 16 + grp, W = a.H * DV;
  const float *__restrict__ pq = a.p + h * DK, *__restrict__ pk = a.p + (a.H + h) * DK, *__restrict__ pv = a.p + 2 * a.H * DK;
  const float *__restrict__ pg = pv + W;
  float *__restrict__ Sc = a.S + ((int64_t)h * DV + c) * DK;
  float4 q[NC], k[NC], s[NC];
#pragma unroll
  for (int i = 0; i < NC; i++) {
    const int e = min(4 * (l + 16 * i), DK - 4);
    s[i] = *(const float4 *)(Sc + e);
    q[i] = *(const float4 *)(pq + e);
    k[i] = *(const float4 *)(pk + e);
  }
  const float v = ct_silu(pv[h * DV + c]), d1 = a.decay[h];
  const int pos = tokpos[1];
  const bool ended = ctrl && ctrl[1] != 0;
  float o = 0.0f;
#pragma unroll
  for (int i = 0; i < NC; i++) {
    const int e = 4 * (l + 16 * i);
    if (e >= DK) continue;
    float4 t = s[i];
    if (pos == 0) t = make_float4(0.f, 0.f, 0.f, 0.f);  // a sequence starts from zero, whatever the one before it left
    // decay S + k v as S + (decay - 1) S + k v: a decay near one keeps all its digits
    t.x = fmaf(t.x, d1, fmaf(ct_silu(k[i].x), v, t.x)), t.y = fmaf(t.y, d1, fmaf(ct_silu(k[i].y), v, t.y));
    t.z = fmaf(t.z, d1, fmaf(ct_silu(k[i].z), v, t.z)), t.w = fmaf(t.w, d1, fmaf(ct_silu(k[i].w), v, t.w));
    o = fmaf(ct_silu(q[i].x), t.x, fmaf(ct_silu(q[i].y), t.y, fmaf(ct_silu(q[i].z), t.z, fmaf(ct_silu(q[i].w), t.w, o))));
    if (!ended) *(float4 *)(Sc + e) = t;
  }
  o = row16_sum(o);
  if (l == 0) agent_store(raw + h * DV + c, o);
  if (!last_ticket(count, nblocks, ticket)) return;
  constexpr int AHEAD = 4;  // pairs of outputs
  float2 x[AHEAD], w[AHEAD], z[AHEAD];
  auto request = [&](int e0) {
#pragma unroll
    for (int b = 0; b < AHEAD; b++) {
      const int e = min(e0 + 512 * b, W - 2);
      x[b] = agent_load2(raw + e), w[b] = *(const float2 *)(a.norm + e), z[b] = *(const float2 *)(pg + e);
    }
  };
  float t = 0.0f;
  for (int e0 = 2 * tid + ((W - 1) / (512 * AHEAD)) * (512 * AHEAD); e0 >= 0; e0 -= 512 * AHEAD) {  // (the first ones last: they stay in registers)
    request(e0);
#pragma unroll
    for (int b = 0; b < AHEAD; b++)
      if (e0 + 512 * b < W) t = fmaf(x[b].x, x[b].x, fmaf(x[b].y, x[b].y, t));
  }
  t = wave_sum(t);
  if (lane == 0) red[wv] = t;
  __syncthreads();
  const float rstd = a.out_scale / sqrtf(((red[0] + red[1]) + (red[2] + red[3])) / (float)(a.H * a.dv) + a.eps);
  for (int e0 = 2 * tid; e0 < W; e0 += 512 * AHEAD) {
    if (e0 != 2 * tid) request(e0);
#pragma unroll
    for (int b = 0; b < AHEAD; b++)
      if (e0 + 512 * b < W)
        *(float2 *)(out + e0 + 512 * b) = make_float2(x[b].x * rstd * w[b].x * ct_sigmoid(z[b].x), x[b].y * rstd * w[b].y * ct_sigmoid(z[b].y));
  }
}

// grid.x: workgroups of a key range; grid.y: the ranges, then as many rows as the lightning workgroups fill
template <int NC, int QB>
__global__ __launch_bounds__(256) void k_parallel_step(WindowArgs w, WindowShape sh, float *__restrict__ wout, LightningArgs n, int nblocks,
                                                       float *__restrict__ nout, ParallelWork k, const int *__restrict__ tokpos,
                                                       const int *__restrict__ ctrl) {
  __shared__ __align__(16) StepLds<NC, QB> S;
  if ((int)blockIdx.y < sh.ranges) {
    window_step<NC, QB>(w, sh, blockIdx.x, blockIdx.y, k.part, k.count + 1, wout, tokpos, S);
  } else {
    const int block = ((int)blockIdx.y - sh.ranges) * (int)gridDim.x + (int)blockIdx.x;
    if (block >= nblocks) return;
    if (n.DK <= 64) lightning_step<1>(n, block, nblocks, k.raw, k.count, nout, tokpos, ctrl, S.red, &S.ticket);
    else if (n.DK <= 128) lightning_step<2>(n, block, nblocks, k.raw, k.count, nout, tokpos, ctrl, S.red, &S.ticket);
    else lightning_step<4>(n, block, nblocks, k.raw, k.count, nout, tokpos, ctrl, S.red, &S.ticket);
  }
}

int launch_parallel_step(const WindowArgs *w, float *wout, const LightningArgs *l, float *lout, const ParallelWork &work, const int *tokpos,
                         const int *ctrl) {
  WindowArgs wa = {};
  LightningArgs la = {};
  WindowShape sh = {};
  int nblocks = 0, pieces = 1, qb = 1;
  if (w) {
    wa = *w;
    sh = window_shape(wa);
    pieces = window_pieces(wa);
    qb = window_qb(wa);
  }
  if (l) {
    la = *l;
    nblocks = la.H * la.DV / 16;
  }
  if (pieces > 4 || la.DK > 256) return fail(CTHIP_E_UNSUPPORTED, "window / lightning attention: heads of more than 256");
  const int gx = w ? sh.heads : nblocks;
  const dim3 grid((unsigned)gx, (unsigned)(sh.ranges + (nblocks + gx - 1) / gx)), b256(256);
#define GO(N, Q) hipLaunchKernelGGL((k_parallel_step<N, Q>), grid, b256, 0, state().stream, wa, sh, wout, la, nblocks, lout, work, tokpos, ctrl)
#define GO_N(N)            \
  if (qb <= 1) GO(N, 1);   \
  else if (qb <= 2) GO(N, 2); \
  else GO(N, 4)
  if (pieces <= 1) { GO_N(1); }
  else if (pieces <= 2) { GO_N(2); }
  else if (qb <= 1) GO(4, 1);
  else GO(4, 2);
#undef GO_N
#undef GO
  CTHIP_LAUNCH_CHECK();
  return 0;
}

}  // namespace cthip
