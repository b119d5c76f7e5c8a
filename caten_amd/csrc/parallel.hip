// A decode step of a layer whose mixers are attention over a sliding window (window.hip), lightning attention
// (lightning.hip), or the two side by side: one launch, whose workgroups belong to one mixer or the other.
//
//   window     workgroup (key range, key/value head, up to QB of its query heads).  It takes the root mean squares of all
//              queries and keys, normalises and rotates its own, and attends over its share of the ring: 16 lanes per row,
//              16 rows a tile, range r of n takes tiles r, r + n, ... .  Rings are walked by row, not by position, so the
//              first rows are asked for before the position is known; which position a row holds follows from it.  The new
//              key and value come from the projection row; the range that owns their row of the ring stores them.
//   lightning  workgroup (head, 16 value columns), 16 lanes per column: the state's rows are read once, updated, read out
//              and written once.  The norm takes all heads' outputs.
//
// What meets across workgroups -- a head's key ranges, the heads' outputs in front of the norm -- is left in memory with
// device-scope stores, a ticket is drawn, and the workgroup with the last ticket finishes (as k_attn_cached does).
#include "common.h"
#include "mixers.h"

namespace cthip {

struct WindowShape {
  int ranges, qgroups, blocks;  // qgroups: workgroups of up to QB query heads per key/value head
};
constexpr int window_qb(int rep) { return rep >= 3 ? 4 : rep; }
static WindowShape window_shape(const WindowArgs &a) {
  const int rep = a.H / a.G, qb = window_qb(rep);
  WindowShape w;
  w.qgroups = (rep + qb - 1) / qb;
  const int tiles = (a.rows + 15) / 16, fill = 512 / (a.G * w.qgroups);
  w.ranges = tiles < kWindowMaxRanges ? tiles : kWindowMaxRanges;
  if (w.ranges > fill) w.ranges = fill < 1 ? 1 : fill;
  w.blocks = w.ranges * w.qgroups * a.G;
  return w;
}
constexpr int part_pitch(int dv) { return dv + 4; }  // a range's record of one head: DV sums, maximum, denominator, two unused
int window_tickets(const WindowArgs &a) { return window_shape(a).qgroups * a.G; }
size_t window_part_floats(const WindowArgs &a) { return (size_t)window_shape(a).blocks * window_qb(a.H / a.G) * part_pitch(a.DV); }
size_t lightning_raw_floats(const LightningArgs &a) { return (size_t)a.H * a.DV + (size_t)a.H * a.DV / 16; }

__device__ __forceinline__ float agent_load(const float *p) { return __hip_atomic_load(p, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT); }
__device__ __forceinline__ void agent_store(float *p, float v) { __hip_atomic_store(p, v, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT); }

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
  float o[4][QB][64 * NC], m[4][QB], l[4][QB];
  float red[8];
  int ticket;
};

// NC: 64-entry pieces of a head, at most; QB: query heads of a workgroup
template <int NC, int QB>
__device__ void window_step(const WindowArgs &a, int nranges, int qgroups, int block, float *__restrict__ part, int *__restrict__ count,
                            float *__restrict__ out, const int *__restrict__ tokpos, StepLds<NC, QB> &S) {
  constexpr int U = NC >= 4 ? 1 : 2;  // tiles a wavefront works on together
  constexpr int QE = (QB * 64 * NC + 255) / 256;
  const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6, g16 = lane >> 4, l = lane & 15;
  const int hg = block % (a.G * qgroups), range = block / (a.G * qgroups), g = hg / qgroups, rep = a.H / a.G;
  const int h0 = g * rep + (hg % qgroups) * QB, nq = min(QB, (g + 1) * rep - h0);  // this workgroup's query heads
  const int DK = a.DK, DV = a.DV, KW = a.G * DK, VW = a.G * DV, QW = a.H * DK, rows = a.rows, half = a.rope ? a.half : 0;
  const float *__restrict__ pq = a.p, *__restrict__ pk = pq + QW, *__restrict__ pv = pk + KW;
  const int pos = tokpos[1];
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
  request(0, range);  // (whatever the position, a range starts with this tile)
  // ---- this step's queries and key ----
  float qa[QE], qb[QE], wa[QE], wb[QE];
#pragma unroll
  for (int j = 0; j < QE; j++) {
    const int it = min(tid + 256 * j, nq * DK - 1), h = it / DK, d = it - h * DK;
    const int mate = d < half ? d + half : d < 2 * half ? d - half : d;
    const int e = (h0 + h) * DK + d, f = (h0 + h) * DK + mate;
    qa[j] = pq[e], qb[j] = pq[f];
    wa[j] = a.qnorm ? a.qnorm[e] : 1.0f, wb[j] = a.qnorm ? a.qnorm[f] : 1.0f;
  }
  const int kd = min(tid, DK - 1), kmate = kd < half ? kd + half : kd < 2 * half ? kd - half : kd;
  const float ka = pk[g * DK + kd], kb = pk[g * DK + kmate];
  const float wka = a.knorm ? a.knorm[g * DK + kd] : 1.0f, wkb = a.knorm ? a.knorm[g * DK + kmate] : 1.0f;
  float4 vn[NC];
#pragma unroll
  for (int i = 0; i < NC; i++) vn[i] = *(const float4 *)(pv + g * DV + min(4 * (l + 16 * i), DV - 4));
  float qs = 1.0f, ks = 1.0f;
  if (a.qnorm) {
    float sq = 0.0f, sk = 0.0f;
    constexpr int SB = 4;
    for (int e0 = 4 * tid; e0 < QW; e0 += 1024 * SB) {
      float4 x[SB];
#pragma unroll
      for (int b = 0; b < SB; b++) x[b] = *(const float4 *)(pq + min(e0 + 1024 * b, QW - 4));
#pragma unroll
      for (int b = 0; b < SB; b++)
        if (e0 + 1024 * b < QW) sq = fmaf(x[b].x, x[b].x, fmaf(x[b].y, x[b].y, fmaf(x[b].z, x[b].z, fmaf(x[b].w, x[b].w, sq))));
    }
    for (int e = 4 * tid; e < KW; e += 1024) {
      const float4 x = *(const float4 *)(pk + e);
      sk = fmaf(x.x, x.x, fmaf(x.y, x.y, fmaf(x.z, x.z, fmaf(x.w, x.w, sk))));
    }
    sq = wave_sum(sq), sk = wave_sum(sk);
    if (lane == 0) S.red[wv] = sq, S.red[4 + wv] = sk;
  }
  const int held = min(pos + 1, rows), tiles = (held + 15) >> 4, nr = min(nranges, (tiles + 1) >> 1);
  if (range >= nr) return;  // (uniform)
#pragma unroll
  for (int u = 1; u < U; u++) request(u, range + nr * u);
  float2 qc[QE], kc = make_float2(1.0f, 0.0f);
#pragma unroll
  for (int j = 0; j < QE; j++) {
    const int d = min(tid + 256 * j, nq * DK - 1) % DK, i = d < half ? d : d - half;
    qc[j] = d < 2 * half ? a.rope[(int64_t)pos * half + i] : make_float2(1.0f, 0.0f);
  }
  if (kd < 2 * half) kc = a.rope[(int64_t)pos * half + (kd < half ? kd : kd - half)];
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
  for (int j = 0; j < QE; j++) {
    const int it = tid + 256 * j;
    if (it < nq * DK) S.q[it / DK][it % DK] = turned(it % DK, qa[j] * qs * wa[j], qb[j] * qs * wb[j], qc[j]);
  }
  if (tid < DK) S.k[tid] = turned(tid, ka * ks * wka, kb * ks * wkb, kc);
  __syncthreads();
  const int cur = pos % rows;
  float4 q[QB][NC], o[QB][NC], kn[NC];
  float m[QB], L[QB];
#pragma unroll
  for (int i = 0; i < NC; i++) {
    const int e = 4 * (l + 16 * i);
    const float4 zero = make_float4(0.f, 0.f, 0.f, 0.f);
    kn[i] = e < DK ? *(const float4 *)&S.k[e] : zero;
#pragma unroll
    for (int h = 0; h < QB; h++) {
      q[h][i] = o[h][i] = zero;
      if (h < nq && e < DK) {
        const float4 t = *(const float4 *)&S.q[h][e];
        q[h][i] = make_float4(t.x * a.scale, t.y * a.scale, t.z * a.scale, t.w * a.scale);
      }
    }
  }
#pragma unroll
  for (int h = 0; h < QB; h++) m[h] = -INFINITY, L[h] = 0.0f;
  if ((cur >> 4) % nr == range && hg % qgroups == 0 && tid < 16) {  // the new row: nobody reads this row of the ring in this step
#pragma unroll
    for (int i = 0; i < NC; i++) {
      const int e = 4 * (l + 16 * i);
      if (e < DK) *(float4 *)(a.K + (int64_t)cur * KW + g * DK + e) = kn[i];
      if (e < DV) *(float4 *)(a.V + (int64_t)cur * VW + g * DV + e) = vn[i];
    }
  }
  for (int tile0 = range; tile0 < tiles; tile0 += U * nr) {
    if (tile0 != range) {
#pragma unroll
      for (int u = 0; u < U; u++) request(u, tile0 + nr * u);
    }
    bool ok[U];
#pragma unroll
    for (int u = 0; u < U; u++) {
      const int slot = (tile0 + nr * u) * 16 + 4 * wv + g16;
      int back = cur - slot;
      back += back < 0 ? rows : 0;
      ok[u] = slot < rows && back <= pos && back < a.window;
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
      float sc[U], top = -INFINITY;
#pragma unroll
      for (int u = 0; u < U; u++) {
        float d = 0.0f;
#pragma unroll
        for (int i = 0; i < NC; i++)
          d = fmaf(q[h][i].x, kr[u][i].x, fmaf(q[h][i].y, kr[u][i].y, fmaf(q[h][i].z, kr[u][i].z, fmaf(q[h][i].w, kr[u][i].w, d))));
        d = row16_sum(d);
        sc[u] = ok[u] ? d : -INFINITY;
        top = fmaxf(top, sc[u]);
      }
      const float m_new = fmaxf(m[h], groups16_max(top));
      const float m_use = m_new == -INFINITY ? 0.0f : m_new;  // no row of this wavefront's yet
      const float corr = ct_exp(m[h] - m_use);
      float ps = 0.0f, pr[U];
#pragma unroll
      for (int u = 0; u < U; u++) {
        pr[u] = ct_exp(sc[u] - m_use);
        ps += pr[u];
      }
      L[h] = fmaf(L[h], corr, groups16_sum(ps));
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
  // the wavefront's four groups of lanes, then the wavefronts through LDS
#pragma unroll
  for (int h = 0; h < QB; h++) {
#pragma unroll
    for (int i = 0; i < NC; i++) {
      float4 t = o[h][i];
      t.x += __shfl_xor(t.x, 16, 64), t.y += __shfl_xor(t.y, 16, 64), t.z += __shfl_xor(t.z, 16, 64), t.w += __shfl_xor(t.w, 16, 64);
      t.x += __shfl_xor(t.x, 32, 64), t.y += __shfl_xor(t.y, 32, 64), t.z += __shfl_xor(t.z, 32, 64), t.w += __shfl_xor(t.w, 32, 64);
      if (g16 == 0) *(float4 *)&S.o[wv][h][4 * (l + 16 * i)] = t;
    }
    if (lane == 0) S.m[wv][h] = m[h], S.l[wv][h] = L[h];
  }
  __syncthreads();
  const int og = QW + KW + VW;  // the gate in the projection row
  auto put = [&](int h, int c, float v) {
    const int e = (h0 + h) * DV + c;
    v *= a.out_scale;
    out[e] = a.gated ? v * ct_sigmoid(a.p[og + e]) : v;
  };
  for (int it = tid; it < nq * DV; it += 256) {
    const int h = it / DV, c = it - h * DV;
    const float M = fmaxf(fmaxf(S.m[0][h], S.m[1][h]), fmaxf(S.m[2][h], S.m[3][h]));
    const float Mu = M == -INFINITY ? 0.0f : M;
    float v = 0.0f, den = 0.0f;
#pragma unroll
    for (int w = 0; w < 4; w++) {
      const float e = ct_exp(S.m[w][h] - Mu);
      v = fmaf(e, S.o[w][h][c], v);
      den = fmaf(e, S.l[w][h], den);
    }
    if (nr == 1) {
      if (a.sink) {
        const float sk = a.sink[h0 + h], top = fmaxf(M, sk), cr = ct_exp(M - top);
        put(h, c, v * cr / fmaf(den, cr, ct_exp(sk - top)));
      } else {
        put(h, c, v / den);
      }
    } else {
      float *rec = part + ((int64_t)(hg * nranges + range) * QB + h) * part_pitch(DV);
      agent_store(rec + c, v);
      if (c == 0) agent_store(rec + DV, M), agent_store(rec + DV + 1, den);
    }
  }
  if (nr == 1) return;
  if (!last_ticket(count + hg, nr, &S.ticket)) return;
  for (int it = tid; it < nq * DV; it += 256) {
    const int h = it / DV, c = it - h * DV;
    const float *rec = part + ((int64_t)hg * nranges * QB + h) * part_pitch(DV);
    const int64_t pitch = (int64_t)QB * part_pitch(DV);
    float mv[kWindowMaxRanges], lv[kWindowMaxRanges], ov[kWindowMaxRanges];
#pragma unroll
    for (int r = 0; r < kWindowMaxRanges; r++) {  // all of them requested before the first is used
      const float *t = rec + min(r, nr - 1) * pitch;
      mv[r] = agent_load(t + DV), lv[r] = agent_load(t + DV + 1), ov[r] = agent_load(t + c);
    }
    float M = a.sink ? a.sink[h0 + h] : -INFINITY;
#pragma unroll
    for (int r = 0; r < kWindowMaxRanges; r++)
      if (r < nr) M = fmaxf(M, mv[r]);
    float v = 0.0f, den = a.sink ? ct_exp(a.sink[h0 + h] - M) : 0.0f;
#pragma unroll
    for (int r = 0; r < kWindowMaxRanges; r++)
      if (r < nr) {
        const float e = ct_exp(mv[r] - M);
        v = fmaf(e, ov[r], v);
        den = fmaf(e, lv[r], den);
      }
    put(h, c, v / den);
  }
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
  const float ss = wave_sum(l == 0 ? o * o : 0.0f);
  if (lane == 0) red[wv] = ss;
  __syncthreads();
  if (tid == 0) agent_store(raw + W + block, (red[0] + red[1]) + (red[2] + red[3]));
  if (!last_ticket(count, nblocks, ticket)) return;
  constexpr int AHEAD = 8;
  float x[AHEAD], w[AHEAD], z[AHEAD];
  auto request = [&](int e0) {
#pragma unroll
    for (int b = 0; b < AHEAD; b++) {
      const int e = min(e0 + 256 * b, W - 1);
      x[b] = agent_load(raw + e), w[b] = a.norm[e], z[b] = pg[e];
    }
  };
  request(tid);
  float t = 0.0f;
  for (int e = tid; e < nblocks; e += 256) t += agent_load(raw + W + e);
  t = wave_sum(t);
  if (lane == 0) red[4 + wv] = t;
  __syncthreads();
  const float rstd = a.out_scale / sqrtf(((red[4] + red[5]) + (red[6] + red[7])) / (float)(a.H * a.dv) + a.eps);
  for (int e0 = tid; e0 < W; e0 += 256 * AHEAD) {
    if (e0 != tid) request(e0);
#pragma unroll
    for (int b = 0; b < AHEAD; b++)
      if (e0 + 256 * b < W) out[e0 + 256 * b] = x[b] * rstd * w[b] * ct_sigmoid(z[b]);
  }
}

template <int NC, int QB>
__global__ __launch_bounds__(256) void k_parallel_step(WindowArgs w, int ranges, int qgroups, int wblocks, float *__restrict__ wout, LightningArgs n,
                                                       int nblocks, float *__restrict__ nout, ParallelWork k, const int *__restrict__ tokpos,
                                                       const int *__restrict__ ctrl) {
  __shared__ __align__(16) StepLds<NC, QB> S;
  if ((int)blockIdx.x < wblocks) window_step<NC, QB>(w, ranges, qgroups, blockIdx.x, k.part, k.count + 1, wout, tokpos, S);
  else lightning_step<NC>(n, blockIdx.x - wblocks, nblocks, k.raw, k.count, nout, tokpos, ctrl, S.red, &S.ticket);
}

int launch_parallel_step(const WindowArgs *w, float *wout, const LightningArgs *l, float *lout, const ParallelWork &work, const int *tokpos,
                         const int *ctrl) {
  WindowArgs wa = {};
  LightningArgs la = {};
  WindowShape sh = {0, 1, 0};
  int nblocks = 0, qb = 1, most = 0;
  if (w) {
    wa = *w;
    sh = window_shape(wa);
    qb = window_qb(wa.H / wa.G);
    most = wa.DK > wa.DV ? wa.DK : wa.DV;
  }
  if (l) {
    la = *l;
    nblocks = la.H * la.DV / 16;
    if (la.DK > most) most = la.DK;
  }
  if (most > 256) return fail(CTHIP_E_UNSUPPORTED, "window / lightning attention: heads of %d (at most 256)", most);
  const dim3 grid((unsigned)(sh.blocks + nblocks)), b256(256);
#define GO(N, Q) hipLaunchKernelGGL((k_parallel_step<N, Q>), grid, b256, 0, state().stream, wa, sh.ranges, sh.qgroups, sh.blocks, wout, la, nblocks, lout, work, tokpos, ctrl)
#define GO_N(N)            \
  if (qb <= 1) GO(N, 1);   \
  else if (qb <= 2) GO(N, 2); \
  else GO(N, 4)
  if (most <= 64) { GO_N(1); }
  else if (most <= 128) { GO_N(2); }
  else { GO_N(4); }
#undef GO_N
#undef GO
  CTHIP_LAUNCH_CHECK();
  return 0;
}

}  // namespace cthip
