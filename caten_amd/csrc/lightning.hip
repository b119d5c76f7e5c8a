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
// on v_mfma_f32_16x16x4_f32 (fp32 products), with a chunk's rows in LDS, where they arrive behind silu.  Operand order as in
// delta.hip: lane l supplies a row's four floats 4 (l/16) .. of a 16-float piece to four matrix instructions, and a result
// tile holds rows 4 (l/16) + i of column l % 16 in register i.
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

__device__ __forceinline__ float4 silu4(const float4 v) {  // (hardware exponential and reciprocal, each within an ulp)
  auto f = [](float x) { return x * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(x * -1.44269504f)); };
  return make_float4(f(v.x), f(v.y), f(v.z), f(v.w));
}
// floats between two rows of n (a multiple of 16) in LDS.  Columns: four consecutive rows of 16 columns meet different
// banks.  Rows: so do 16-byte pieces of consecutive rows, and columns of rows that are four apart.
__host__ __device__ constexpr int column_pitch(int n) { return (n & 16) ? n : n + 16; }
__host__ __device__ constexpr int row_pitch(int n) { return n + 4; }

// A chunk's rows of n <= 256 floats on their way to LDS, through the registers of 512 threads: 16 threads a row
struct RowTile {
  float4 x[2][4];
  __device__ __forceinline__ void load(const float *__restrict__ src, int64_t ld, int n, int last) {  // rows past `last` repeat it
#pragma unroll
    for (int r = 0; r < 2; r++)
#pragma unroll
      for (int c = 0; c < 4; c++) {
        const int j = ((int)threadIdx.x >> 4) + 32 * r, e = 4 * (((int)threadIdx.x & 15) + 16 * c);
        if (e < n) x[r][c] = *(const float4 *)(src + (int64_t)min(j, last) * ld + e);
      }
  }
  template <typename Scale>
  __device__ __forceinline__ void put(float *__restrict__ lds, int pitch, int n, Scale scale) const {  // row j behind silu, times scale(j)
#pragma unroll
    for (int r = 0; r < 2; r++) {
      const int j = ((int)threadIdx.x >> 4) + 32 * r;
      const float f = scale(j);
#pragma unroll
      for (int c = 0; c < 4; c++) {
        const int e = 4 * (((int)threadIdx.x & 15) + 16 * c);
        if (e < n) {
          const float4 v = silu4(x[r][c]);
          *(float4 *)(lds + j * pitch + e) = make_float4(v.x * f, v.y * f, v.z * f, v.w * f);
        }
      }
    }
  }
};

// Workgroup (chunk, head); wavefront w takes the key tiles w, w + 8, ... against every value tile.
template <int NV>  // 16-column value tiles, at most
__global__ __launch_bounds__(512) void k_lightning_local(LightningArgs a, const float *__restrict__ p, float *__restrict__ U, int s) {
  extern __shared__ __align__(16) float light_lds[];
  const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6, lo = lane & 15, hi = lane >> 4;
  const int c0 = blockIdx.x * kLightChunk, h = blockIdx.y, DK = a.DK, DV = a.DV, nv = DV >> 4, kp = column_pitch(DK), vp = column_pitch(DV);
  const int last = min(kLightChunk, s - c0) - 1;
  const float lg = a.decay[a.H + h];
  float *__restrict__ K = light_lds, *__restrict__ V = light_lds + kLightChunk * kp;
  const float *__restrict__ pk = p + (int64_t)c0 * a.ldp + (int64_t)(a.H + h) * DK, *__restrict__ pv = p + (int64_t)c0 * a.ldp + 2 * (int64_t)a.H * DK + (int64_t)h * DV;
  RowTile kx, vx;
  kx.load(pk, a.ldp, DK, last);
  vx.load(pv, a.ldp, DV, last);
  kx.put(K, kp, DK, [&](int j) { return j <= last ? exp2f((float)(last - j) * lg) : 0.0f; });
  vx.put(V, vp, DV, [](int) { return 1.0f; });
  __syncthreads();
  float *__restrict__ Uh = U + ((int64_t)blockIdx.x * a.H + h) * DV * DK;
  for (int kt = wv; kt < (DK >> 4); kt += 8) {
    v4f_t acc[NV];
#pragma unroll
    for (int v = 0; v < NV; v++) acc[v] = v4f_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (int j = 0; j < kLightChunk; j += 4) {  // lane (lo, hi): token j + hi
      const float kj = K[(j + hi) * kp + 16 * kt + lo];
#pragma unroll
      for (int v = 0; v < NV; v++) acc[v] = __builtin_amdgcn_mfma_f32_16x16x4f32(kj, V[(j + hi) * vp + 16 * min(v, nv - 1) + lo], acc[v], 0, 0, 0);
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

// Workgroup (chunk, head).  The ten 16 x 16 tiles on and below the diagonal of P_ij = decay^(i - j) (q_i . k_j) go round the
// wavefronts and through LDS; then wavefront w takes the value tiles w, w + 8, ... of all rows.  K and V share their place.
template <int NK>  // 16-entry pieces of a key, at most
__global__ __launch_bounds__(512) void k_lightning_out(LightningArgs a, const float *__restrict__ p, const float *__restrict__ U, float *__restrict__ out,
                                                       int64_t ldo, int s) {
  constexpr int PP = kLightChunk + 4;
  extern __shared__ __align__(16) float light_lds[];
  const int tid = threadIdx.x, lane = tid & 63, wv = tid >> 6, lo = lane & 15, hi = lane >> 4;
  const int c0 = blockIdx.x * kLightChunk, h = blockIdx.y, DK = a.DK, DV = a.DV, nk = DK >> 4, nv = DV >> 4, qp = row_pitch(DK), vp = row_pitch(DV);
  const int last = min(kLightChunk, s - c0) - 1;
  const float lg = a.decay[a.H + h];
  float *__restrict__ P = light_lds, *__restrict__ Q = P + kLightChunk * PP, *__restrict__ KV = Q + kLightChunk * qp;
  const float *__restrict__ p0 = p + (int64_t)c0 * a.ldp;
  const float *__restrict__ S = U + ((int64_t)blockIdx.x * a.H + h) * DV * DK;
  float4 sn[NK];  // the state of a value tile, requested a tile ahead
  auto request = [&](int vt) {
#pragma unroll
    for (int c = 0; c < NK; c++) sn[c] = *(const float4 *)(S + (int64_t)(16 * min(vt, nv - 1) + lo) * DK + 16 * min(c, nk - 1) + 4 * hi);
  };
  request(wv);
  auto one = [](int) { return 1.0f; };
  RowTile qx, kx;
  qx.load(p0 + (int64_t)h * DK, a.ldp, DK, last);
  kx.load(p0 + (int64_t)(a.H + h) * DK, a.ldp, DK, last);
  qx.put(Q, qp, DK, one);
  kx.put(KV, qp, DK, one);
  kx.load(p0 + 2 * (int64_t)a.H * DK + (int64_t)h * DV, a.ldp, DV, last);  // (the values)
  __syncthreads();
  for (int i = wv; i < 10; i += 8) {
    const int rt = i < 1 ? 0 : i < 3 ? 1 : i < 6 ? 2 : 3, kt = i - rt * (rt + 1) / 2;
    v4f_t acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (int c = 0; c < nk; c++)
      acc = mfma4(*(const float4 *)(KV + (16 * kt + lo) * qp + 16 * c + 4 * hi), vec4(*(const float4 *)(Q + (16 * rt + lo) * qp + 16 * c + 4 * hi)), acc);
    float w[4];  // key 16 kt + 4 hi + t of query 16 rt + lo
#pragma unroll
    for (int t = 0; t < 4; t++) {
      const int d = 16 * (rt - kt) + lo - 4 * hi - t;
      w[t] = d >= 0 ? acc[t] * exp2f((float)d * lg) : 0.0f;
    }
    *(float4 *)(P + (16 * rt + lo) * PP + 16 * kt + 4 * hi) = make_float4(w[0], w[1], w[2], w[3]);
  }
  __syncthreads();
  kx.put(KV, vp, DV, one);
  __syncthreads();
  float g[4][4];  // decay^(i + 1) of row i = 16 r + 4 hi + t
#pragma unroll
  for (int r = 0; r < 4; r++)
#pragma unroll
    for (int t = 0; t < 4; t++) g[r][t] = exp2f((float)(16 * r + 4 * hi + t + 1) * lg);
  for (int vt = wv; vt < nv; vt += 8) {
    v4f_t o[4];
#pragma unroll
    for (int r = 0; r < 4; r++) o[r] = v4f_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int c = 0; c < NK; c++) {
      const v4f_t sv = vec4(sn[c]);
      if (c < nk)
#pragma unroll
        for (int r = 0; r < 4; r++) o[r] = mfma4(*(const float4 *)(Q + (16 * r + lo) * qp + 16 * c + 4 * hi), sv, o[r]);
    }
    if (vt + 8 < nv) request(vt + 8);
#pragma unroll
    for (int r = 0; r < 4; r++)
#pragma unroll
      for (int t = 0; t < 4; t++) o[r][t] *= g[r][t];
#pragma unroll
    for (int kt = 0; kt < 4; kt++) {
      v4f_t v;
#pragma unroll
      for (int t = 0; t < 4; t++) v[t] = KV[(16 * kt + 4 * hi + t) * vp + 16 * vt + lo];
#pragma unroll
      for (int r = kt; r < 4; r++) o[r] = mfma4(*(const float4 *)(P + (16 * r + lo) * PP + 16 * kt + 4 * hi), v, o[r]);
    }
#pragma unroll
    for (int r = 0; r < 4; r++)
#pragma unroll
      for (int t = 0; t < 4; t++) {
        const int i = 16 * r + 4 * hi + t;
        if (i <= last) out[(int64_t)(c0 + i) * ldo + (int64_t)h * DV + 16 * vt + lo] = o[r][t];
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

int launch_lightning_rows(const LightningArgs &a, float *out, int64_t ldo, int s, int n, float *scratch) {
  if (s <= 0) return 0;
  if (a.DK > 256 || a.DV > 256) return fail(CTHIP_E_UNSUPPORTED, "lightning attention: heads of %d / %d (at most 256)", a.DK, a.DV);
  hipStream_t st = state().stream;
  const dim3 b256(256);
  const size_t lds_local = sizeof(float) * kLightChunk * (size_t)(column_pitch(a.DK) + column_pitch(a.DV));
  const size_t lds_out = sizeof(float) * kLightChunk * (size_t)(kLightChunk + 4 + row_pitch(a.DK) + row_pitch(a.DK > a.DV ? a.DK : a.DV));
  const int64_t quads = (int64_t)a.H * a.DV * a.DK / 4;
  for (int t0 = 0; t0 < s; t0 += kLightChunk * kLightSegment) {
    const int m = s - t0 < kLightChunk * kLightSegment ? s - t0 : kLightChunk * kLightSegment;
    const float *pt = a.p + (int64_t)t0 * a.ldp;
    float *ot = out + (int64_t)t0 * ldo;
    const dim3 grid((unsigned)((m + kLightChunk - 1) / kLightChunk), (unsigned)a.H);
#define GO(KERNEL, BYTES, ...)                                                                                                     \
  do {                                                                                                                             \
    static const hipError_t large = hipFuncSetAttribute((const void *)KERNEL, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024); \
    CTHIP_CHECK(large);                                                                                                            \
    hipLaunchKernelGGL(KERNEL, grid, dim3(512), BYTES, st, a, pt, scratch, __VA_ARGS__);                                                \
  } while (0)
#define LOCAL(N) GO(k_lightning_local<N>, lds_local, m)
#define OUT(N) GO(k_lightning_out<N>, lds_out, ot, ldo, m)
    if (a.DV <= 32) LOCAL(2);
    else if (a.DV <= 64) LOCAL(4);
    else if (a.DV <= 128) LOCAL(8);
    else LOCAL(16);
    hipLaunchKernelGGL(k_lightning_carry, dim3((unsigned)((quads + 255) / 256)), b256, 0, st, a, scratch, m, n + t0);
    if (a.DK <= 32) OUT(2);
    else if (a.DK <= 64) OUT(4);
    else if (a.DK <= 128) OUT(8);
    else OUT(16);
#undef GO
#undef LOCAL
#undef OUT
    CTHIP_LAUNCH_CHECK();
  }
  hipLaunchKernelGGL(k_lightning_finish, dim3((unsigned)s), b256, 0, st, a, a.p, out, ldo);
  CTHIP_LAUNCH_CHECK();
  return 0;
}

}  // namespace cthip
