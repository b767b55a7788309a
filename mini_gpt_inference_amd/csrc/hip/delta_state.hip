// The gated delta rule: linear attention whose float32 state per request and head, before it takes a token's
// value in, first gives up what it already holds under the token's key.
//
//   S <- g_t S;   u_t = beta_t (v_t - S^T k_t);   S <- S + k_t u_t^T;   o_t = S^T q_t      (S: [D, E])
//
// with g_t = exp(-exp(a_log_h) softplus(a_t[h] + dt_bias_h)) and beta_t = sigmoid(b_t[h]), one number per head,
// and unit queries and keys x / sqrt(sum(x^2) + 1e-6), the queries also times q_scale.  Heads share queries and
// keys in groups (head h reads group h / heads_per_group), values are per head.  Queries, keys and values lie in
// rows of `x`, the two logits per head in rows of `z`.  S is zero before a request's first token and comes from,
// and goes back to, the request's slot of a float32 pool; everything from the loaded numbers on is float32.
#include "common.h"
#include "dtype_io.h"
#include "launchers.h"

#define DS_MAX 256     // largest D and E
#define DS_TC 8        // tokens staged at once
#define DS_UNIT_EPS 1e-6f
#define DS_LOG2E 1.4426950408889634f

__device__ __forceinline__ float ds_softplus(float v) { return fmaxf(v, 0.f) + log1pf(expf(-fabsf(v))); }
__device__ __forceinline__ float ds_sigmoid(float v) { return 1.0f / (1.0f + expf(-v)); }

// sum over lanes l, l ^ 16, l ^ 32, l ^ 48, the same in all four
__device__ __forceinline__ float ds_sum_rows(float v) {
  const unsigned int u = __float_as_uint(v);
  const auto a = __builtin_amdgcn_permlane16_swap(u, u, false, false);
  const float x = __uint_as_float(a[0]) + __uint_as_float(a[1]);
  const unsigned int ux = __float_as_uint(x);
  const auto b = __builtin_amdgcn_permlane32_swap(ux, ux, false, false);
  return __uint_as_float(b[0]) + __uint_as_float(b[1]);
}

// ---------------------------------------------------------------------------------------------
// Token by token: one workgroup per (request, head), a wave per 16 value channels.  A wave's lane (dg, ec) owns
// S[d][ec] for the rows d of quarter dg, in registers, so the sums over d meet inside the wave.  Both products
// with S are taken of the decayed state before the write, o = S^T q + (q . k) u, so a token costs one meeting.
// With `gate_off` >= 0 each head's output is then divided by its root mean square over E (eps), multiplied by
// norm_w and by silu of the gate's row (in z, head by head), and stored in the rows' type; otherwise o is stored
// as float32.
template <typename T, int DQ, int THREADS>     // DQ: rows of S a lane holds at most; THREADS: of the workgroup, at most
__global__ __launch_bounds__(THREADS) void delta_state_kernel(
    const T* __restrict__ x, long ldx, int q_off, int k_off, int v_off, const T* __restrict__ z, long ldz, int b_off,
    int a_off, int gate_off, int n_head, int heads_per_group, int D, int E, float q_scale,
    const float* __restrict__ dt_bias, const float* __restrict__ a_log, const float* __restrict__ norm_w, float eps,
    float* __restrict__ state, long ld_state, const int* __restrict__ state_slots, const int* __restrict__ cu_q,
    const int* __restrict__ positions, void* __restrict__ out, long ldo) {
  constexpr int LDQ = DQ + 4;            // a quarter's stretch of a staged row
  __shared__ __attribute__((aligned(16))) float q_s[DS_TC][4 * LDQ], k_s[DS_TC][4 * LDQ];
  __shared__ float v_s[DS_TC][DS_MAX], o_s[DS_TC][DS_MAX], gate_s[DS_TC][DS_MAX], g_s[DS_TC], beta_s[DS_TC], qk_s[DS_TC];
  const int r = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int slot = state_slots[r];
  const int t_begin = cu_q[r], t_end = cu_q[r + 1];
  if (slot < 0 || t_end <= t_begin) return;     // a request of the padding
  const int wave = tid >> 6, lane = tid & 63, n_waves = blockDim.x >> 6;
  const int dg = lane >> 4, c = wave * 16 + (lane & 15);
  const int quarter = (D + 3) >> 2, d0 = dg * quarter;
  const int rows = D - d0 < quarter ? D - d0 : quarter;      // may be <= 0
  const int group = h / heads_per_group;
  const bool mine = c < E;
  const bool fresh = positions[t_begin] == 0;   // the request's first token: its state starts at zero
  float* st = state + (long)slot * ld_state + (long)h * D * E;
  float S[DQ];
#pragma unroll
  for (int j = 0; j < DQ; ++j) S[j] = (mine && !fresh && j < rows) ? st[(long)(d0 + j) * E + c] : 0.f;
  const float rate = expf(a_log[h]), bias = dt_bias[h];
  const int staged = t_end - t_begin < DS_TC ? t_end - t_begin : DS_TC;
  for (int i = tid; i < staged * 4 * LDQ; i += blockDim.x) {     // rows behind a quarter's last stay zero
    (&q_s[0][0])[i] = 0.f;
    (&k_s[0][0])[i] = 0.f;
  }

  for (int t0 = t_begin; t0 < t_end; t0 += DS_TC) {
    const int nt = t_end - t0 < DS_TC ? t_end - t0 : DS_TC;
    __syncthreads();     // the tokens before are done with
    for (int tt = wave; tt < nt; tt += n_waves) {
      const T* xr = x + (long)(t0 + tt) * ldx + (long)group * D;
      float qv[DS_MAX / 64], kv[DS_MAX / 64];
      float sq = 0.f, sk = 0.f, qk = 0.f;
#pragma unroll
      for (int u = 0; u < DS_MAX / 64; ++u) {
        const int d = lane + 64 * u;
        qv[u] = d < D ? to_float<T>(xr[q_off + d]) : 0.f;
        kv[u] = d < D ? to_float<T>(xr[k_off + d]) : 0.f;
      }
#pragma unroll
      for (int u = 0; u < DS_MAX / 64; ++u) {
        sq = fmaf(qv[u], qv[u], sq);
        sk = fmaf(kv[u], kv[u], sk);
        qk = fmaf(qv[u], kv[u], qk);
      }
      const float iq = q_scale / sqrtf(wave_sum(sq) + DS_UNIT_EPS), ik = 1.0f / sqrtf(wave_sum(sk) + DS_UNIT_EPS);
      qk = wave_sum(qk);
#pragma unroll
      for (int u = 0; u < DS_MAX / 64; ++u) {
        const int d = lane + 64 * u;
        if (d < D) {
          const int at = d / quarter * LDQ + d % quarter;
          q_s[tt][at] = qv[u] * iq;
          k_s[tt][at] = kv[u] * ik;
        }
      }
      if (lane == 0) {
        const T* zr = z + (long)(t0 + tt) * ldz;
        beta_s[tt] = ds_sigmoid(to_float<T>(zr[b_off + h]));
        g_s[tt] = expf(-rate * ds_softplus(to_float<T>(zr[a_off + h]) + bias));
        qk_s[tt] = qk * iq * ik;
      }
    }
    for (int i = tid; i < nt * E; i += blockDim.x) {
      const int tt = i / E, e = i - tt * E;
      v_s[tt][e] = to_float<T>(x[(long)(t0 + tt) * ldx + v_off + (long)h * E + e]);
      if (gate_off >= 0) gate_s[tt][e] = to_float<T>(z[(long)(t0 + tt) * ldz + gate_off + (long)h * E + e]);
    }
    __syncthreads();
    for (int tt = 0; tt < nt; ++tt) {
      const float* kq = &k_s[tt][dg * LDQ];
      const float* qq = &q_s[tt][dg * LDQ];
      const float g = g_s[tt];
      float pk = 0.f, pq = 0.f;
#pragma unroll
      for (int j = 0; j < DQ; j += 4) {
        const float4 k4 = *reinterpret_cast<const float4*>(kq + j), q4 = *reinterpret_cast<const float4*>(qq + j);
        S[j] *= g; S[j + 1] *= g; S[j + 2] *= g; S[j + 3] *= g;
        pk = fmaf(S[j], k4.x, pk); pk = fmaf(S[j + 1], k4.y, pk); pk = fmaf(S[j + 2], k4.z, pk); pk = fmaf(S[j + 3], k4.w, pk);
        pq = fmaf(S[j], q4.x, pq); pq = fmaf(S[j + 1], q4.y, pq); pq = fmaf(S[j + 2], q4.z, pq); pq = fmaf(S[j + 3], q4.w, pq);
      }
      pk = ds_sum_rows(pk);
      pq = ds_sum_rows(pq);
      const float u = mine ? beta_s[tt] * (v_s[tt][c] - pk) : 0.f;
#pragma unroll
      for (int j = 0; j < DQ; j += 4) {
        const float4 k4 = *reinterpret_cast<const float4*>(kq + j);
        S[j] = fmaf(k4.x, u, S[j]); S[j + 1] = fmaf(k4.y, u, S[j + 1]);
        S[j + 2] = fmaf(k4.z, u, S[j + 2]); S[j + 3] = fmaf(k4.w, u, S[j + 3]);
      }
      if (dg == 0 && mine) o_s[tt][c] = fmaf(qk_s[tt], u, pq);
    }
    __syncthreads();
    for (int tt = wave; tt < nt; tt += n_waves) {
      const long orow = (long)(t0 + tt) * ldo + (long)h * E;
      if (gate_off < 0) {
        for (int e = lane; e < E; e += 64) ((float*)out)[orow + e] = o_s[tt][e];
        continue;
      }
      float ov[DS_MAX / 64], gv[DS_MAX / 64], ss = 0.f;
#pragma unroll
      for (int u = 0; u < DS_MAX / 64; ++u) {
        const int e = lane + 64 * u;
        ov[u] = e < E ? o_s[tt][e] : 0.f;
        gv[u] = e < E ? gate_s[tt][e] : 0.f;
        ss = fmaf(ov[u], ov[u], ss);
      }
      const float inv = 1.0f / sqrtf(wave_sum(ss) / (float)E + eps);
#pragma unroll
      for (int u = 0; u < DS_MAX / 64; ++u) {
        const int e = lane + 64 * u;
        if (e < E) ((T*)out)[orow + e] = from_float<T>(ov[u] * inv * norm_w[e] * (gv[u] * ds_sigmoid(gv[u])));
      }
    }
  }
#pragma unroll
  for (int j = 0; j < DQ; ++j)
    if (mine && j < rows) st[(long)(d0 + j) * E + c] = S[j];
}

// x: rows in `dtype` with q at q_off and k at k_off, group by group (D channels each), v at v_off head by head (E
// channels each).  z: rows in the same dtype with the logits of beta at b_off and of the decay at a_off, one per
// head, and, with gate_off >= 0, the heads' gates at gate_off; norm_w: float32 [E].  state: rows of ld_state
// floats, a request's [heads, D, E] at the row of its slot.  out: with gate_off >= 0 rows in `dtype`, else float32.
extern "C" int mgpt_delta_state(const void* x, int dtype, long ldx, int q_off, int k_off, int v_off, const void* z,
                                long ldz, int b_off, int a_off, int gate_off, int n_head, int n_group, int head_dim,
                                int value_dim, float q_scale, const float* dt_bias, const float* a_log,
                                const float* norm_w, float eps, float* state, long ld_state, const int* state_slots,
                                const int* cu_q, int n_req, const int* positions, void* out, long ldo,
                                hipStream_t stream) {
  if (n_req == 0) return MGPT_OK;
  if (!x || !z || !dt_bias || !a_log || !state || !state_slots || !cu_q || !positions || !out ||
      (gate_off >= 0 && !norm_w))
    return MGPT_ERR_NULL;
  if (!dtype_ok(dtype)) return MGPT_ERR_BAD_DTYPE;
  const int D = head_dim, E = value_dim;
  if (n_req < 0 || n_head <= 0 || n_group <= 0 || n_head % n_group || D <= 0 || E <= 0 || D > DS_MAX || E > DS_MAX ||
      ld_state < (long)n_head * D * E)
    return MGPT_ERR_BAD_SHAPE;
  if (n_head > 65535) return MGPT_ERR_TOO_LARGE;
  const int quarter = (D + 3) / 4;
  dim3 grid(n_req, n_head), block(64 * ((E + 15) / 16));
#define DS_LAUNCH3(T, Q, N)                                                                                              \
  hipLaunchKernelGGL((delta_state_kernel<T, Q, N>), grid, block, 0, stream, (const T*)x, ldx, q_off, k_off, v_off,       \
                     (const T*)z, ldz, b_off, a_off, gate_off, n_head, n_head / n_group, D, E, q_scale, dt_bias, a_log, \
                     norm_w, eps, state, ld_state, state_slots, cu_q, positions, out, ldo)
#define DS_LAUNCH2(T, Q)                 \
  {                                      \
    if (E <= 128) DS_LAUNCH3(T, Q, 512); \
    else DS_LAUNCH3(T, Q, 1024);         \
  }
#define DS_LAUNCH(Q)                     \
  {                                      \
    if (dtype == MGPT_F32) DS_LAUNCH2(float, Q) \
    else DS_LAUNCH2(bf16_t, Q)           \
  }
  if (quarter <= 4) DS_LAUNCH(4)
  else if (quarter <= 8) DS_LAUNCH(8)
  else if (quarter <= 16) DS_LAUNCH(16)
  else if (quarter <= 32) DS_LAUNCH(32)
  else DS_LAUNCH(64)
#undef DS_LAUNCH
#undef DS_LAUNCH2
#undef DS_LAUNCH3
  return mgpt_last_error();
}

// ---------------------------------------------------------------------------------------------
// Prompt portions: the recurrence a chunk of 32 tokens at a time, as matrix products on the float32 matrix cores
// (v_mfma_f32_16x16x4_f32: true 32-bit products and sums).  Over a chunk's tokens i = 0 .. n-1, with
// M[i][j] = g_(j+1) ... g_i and G_i = g_0 ... g_i:
//
//   u_i = beta_i (v_i - G_i S^T k_i - sum_(j<i) M[i][j] (k_i . k_j) u_j)
//
// is a triangular system (I + A) U = beta (V - G K S), A[i][j] = beta_i M[i][j] (k_i . k_j) for j < i.  With
// R = (I + A)^-1, W = R diag(beta G) K and U0 = R diag(beta) V:
//
//   U = U0 - W S;   O = diag(G) Q S + P U,  P[i][j] = M[i][j] (q_i . k_j) for j <= i;
//   S <- G_(n-1) S + (diag(M[n-1][.]) K)^T U
//
// Everything but the three lines of the recurrence itself is the same for all value channels and needs no state:
// delta_prepare_kernel makes it for all chunks side by side, one workgroup per (chunk, head), and leaves per
// (chunk, head) one image in the layout in which delta_chunk_kernel wants it in LDS, rows of 16 bytes' multiples:
//   W [32][ld], diag(G) Q [32][ld], (diag(M[n-1][.]) K)^T [Dp][LDP], P [32][LDP] (P[0][32]: G_(n-1)),
// ld = Dp + 4, Dp = D in steps of 16; U0 goes into the rows that will hold the outputs.  Every decay is a product
// over exactly the tokens it spans (a sum of logarithms from j + 1 on, never a difference of two sums).
//
// Chunks of request r have the numbers first(r), first(r) + 1, .. with first(r) = cu_q[r] / 32 + r, which leaves
// room for all of its chunks whatever its length.

#define DC_C 32        // tokens a chunk
#define DC_DMAX 128    // largest D of this path
#define DC_LDP (DC_C + 4)

typedef float ds_f32x4 __attribute__((ext_vector_type(4)));

__device__ __forceinline__ float ds_exp2(float v) { return __builtin_amdgcn_exp2f(v); }

__host__ __device__ __forceinline__ int ds_image_floats(int Dp) {
  return 2 * DC_C * (Dp + 4) + Dp * DC_LDP + DC_C * DC_LDP;
}

__device__ __forceinline__ void ds_load8(const float* p, float (&v)[8]) {
  const ds_f32x4 a = *reinterpret_cast<const ds_f32x4*>(p), b = *reinterpret_cast<const ds_f32x4*>(p + 4);
#pragma unroll
  for (int e = 0; e < 4; ++e) {
    v[e] = a[e];
    v[4 + e] = b[e];
  }
}
__device__ __forceinline__ void ds_load8(const bf16_t* p, float (&v)[8]) {
  const uint4 a = *reinterpret_cast<const uint4*>(p);
  const unsigned words[4] = {a.x, a.y, a.z, a.w};
#pragma unroll
  for (int k = 0; k < 4; ++k) {
    v[2 * k] = __uint_as_float(words[k] << 16);
    v[2 * k + 1] = __uint_as_float(words[k] & 0xffff0000u);
  }
}

// VEC: D is a multiple of 8 and the rows of x are aligned for loads of eight elements
template <typename T, bool VEC>
__global__ __launch_bounds__(256) void delta_prepare_kernel(
    const T* __restrict__ x, long ldx, int q_off, int k_off, int v_off, const T* __restrict__ z, long ldz, int b_off,
    int a_off, int n_head, int heads_per_group, int D, int E, float q_scale, const float* __restrict__ dt_bias,
    const float* __restrict__ a_log, const int* __restrict__ cu_q, int n_req, float* __restrict__ images,
    float* __restrict__ out, long ldo) {
  extern __shared__ __attribute__((aligned(16))) float dc_lds[];
  const int Dp = (D + 15) & ~15, ld = Dp + 4;
  float* Qs = dc_lds;                     // [32][ld] unit queries (scaled)
  float* Ks = Qs + DC_C * ld;             // [32][ld] unit keys
  float* As = Ks + DC_C * ld;             // [32][LDP] k . k, then A
  float* Ps = As + DC_C * DC_LDP;         // [32][LDP] q . k
  float* Ms = Ps + DC_C * DC_LDP;         // [32][LDP] the decays between tokens
  float* Rs = Ms + DC_C * DC_LDP;         // [32][LDP] R
  float* Xs = Ps;                         // [16][LDP] scratch of the block inverse (q . k is in the image by then)
  __shared__ float beta_s[DC_C], l_s[DC_C], G_s[DC_C], bg_s[DC_C];
  const int chunk = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
  const int wave = tid >> 6, lane = tid & 63, r16 = lane & 15, g4 = lane >> 4;
  // the request whose chunks this number belongs to: first() rises with r
  int r = -1;
  for (int s0 = 0; s0 < n_req; s0 += 256) {
    const int s = s0 + tid;
    r += __syncthreads_count(s < n_req && cu_q[s < n_req ? s : 0] / DC_C + s <= chunk);
  }
  if (r < 0) return;
  const int t0 = cu_q[r] + (chunk - (cu_q[r] / DC_C + r)) * DC_C, t_end = cu_q[r + 1];
  if (t0 >= t_end) return;      // a number without a chunk
  const int nt = t_end - t0 < DC_C ? t_end - t0 : DC_C;
  const int group = h / heads_per_group;

  // ---- unit queries and keys: eight threads a token
  {
    const int row = tid >> 3, sub = tid & 7;
    const T* xr = x + (long)(t0 + row) * ldx + (long)group * D;
    float qv[DC_DMAX / 8], kv[DC_DMAX / 8];
    float sq = 0.f, sk = 0.f;
    // value u of a thread is channel sub + 8 u, or (VEC) channel 8 sub + u % 8 + 64 (u / 8)
    auto channel = [&](int u) { return VEC ? 8 * sub + (u & 7) + 64 * (u >> 3) : sub + 8 * u; };
    if (VEC) {
#pragma unroll
      for (int u = 0; u < DC_DMAX / 64; ++u) {
        const int d = 8 * sub + 64 * u;
        float q8[8] = {}, k8[8] = {};
        if (row < nt && d < D) {
          ds_load8(xr + q_off + d, q8);
          ds_load8(xr + k_off + d, k8);
        }
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          qv[8 * u + e] = q8[e];
          kv[8 * u + e] = k8[e];
        }
      }
    } else {
#pragma unroll
      for (int u = 0; u < DC_DMAX / 8; ++u) {
        const int d = channel(u);
        const bool ok = row < nt && d < D;
        qv[u] = ok ? to_float<T>(xr[q_off + d]) : 0.f;
        kv[u] = ok ? to_float<T>(xr[k_off + d]) : 0.f;
      }
    }
#pragma unroll
    for (int u = 0; u < DC_DMAX / 8; ++u) {
      sq = fmaf(qv[u], qv[u], sq);
      sk = fmaf(kv[u], kv[u], sk);
    }
#pragma unroll
    for (int off = 1; off < 8; off <<= 1) {
      sq += __shfl_xor(sq, off);
      sk += __shfl_xor(sk, off);
    }
    const float iq = q_scale / sqrtf(sq + DS_UNIT_EPS), ik = 1.0f / sqrtf(sk + DS_UNIT_EPS);
#pragma unroll
    for (int u = 0; u < DC_DMAX / 8; ++u) {
      const int d = channel(u);
      if (d < Dp) {
        Qs[row * ld + d] = qv[u] * iq;
        Ks[row * ld + d] = kv[u] * ik;
      }
    }
  }
  if (tid < DC_C) {
    float l = 0.f, beta = 0.f;
    if (tid < nt) {
      const T* zr = z + (long)(t0 + tid) * ldz;
      beta = ds_sigmoid(to_float<T>(zr[b_off + h]));
      l = -expf(a_log[h]) * ds_softplus(to_float<T>(zr[a_off + h]) + dt_bias[h]) * DS_LOG2E;
    }
    beta_s[tid] = beta;
    l_s[tid] = l;
  }
  __syncthreads();
  // ---- wave 0: the decays between tokens, a column a lane; waves 1 to 3: k . k and q . k, a 16 x 16 tile each
  if (wave == 0) {
    if (lane <= DC_C) {
      // lane j: tokens j + 1 .. i; lane 32: the whole chunk up to i
      float run = 0.f;
      for (int i = 0; i < DC_C; ++i) {
        if (lane == DC_C || i > lane) run += l_s[i];
        const float m = ds_exp2(run);
        if (lane == DC_C) G_s[i] = m;
        else Ms[i * DC_LDP + lane] = m;      // (above the diagonal: 1, never read)
      }
    }
  } else {
    const int ti = wave == 1 ? 0 : 1, tj = wave == 3 ? 1 : 0;
    ds_f32x4 kk = {0.f, 0.f, 0.f, 0.f}, qk = {0.f, 0.f, 0.f, 0.f};
    for (int k0 = 0; k0 < Dp; k0 += 16) {
      const ds_f32x4 ka = *reinterpret_cast<const ds_f32x4*>(Ks + (ti * 16 + r16) * ld + k0 + 4 * g4);
      const ds_f32x4 qa = *reinterpret_cast<const ds_f32x4*>(Qs + (ti * 16 + r16) * ld + k0 + 4 * g4);
      const ds_f32x4 kb = *reinterpret_cast<const ds_f32x4*>(Ks + (tj * 16 + r16) * ld + k0 + 4 * g4);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        kk = __builtin_amdgcn_mfma_f32_16x16x4f32(ka[e], kb[e], kk, 0, 0, 0);
        qk = __builtin_amdgcn_mfma_f32_16x16x4f32(qa[e], kb[e], qk, 0, 0, 0);
      }
    }
#pragma unroll
    for (int v = 0; v < 4; ++v) {
      As[(ti * 16 + 4 * g4 + v) * DC_LDP + tj * 16 + r16] = kk[v];
      Ps[(ti * 16 + 4 * g4 + v) * DC_LDP + tj * 16 + r16] = qk[v];
    }
  }
  __syncthreads();
  float* img = images + ((long)chunk * n_head + h) * ds_image_floats(Dp);
  float* imgW = img;
  float* imgQ = imgW + DC_C * ld;
  float* imgK = imgQ + DC_C * ld;
  float* imgP = imgK + Dp * DC_LDP;
  for (int e = tid; e < DC_C * DC_C; e += 256) {
    const int i = e >> 5, j = e & 31;
    const float m = Ms[i * DC_LDP + j];
    As[i * DC_LDP + j] = j < i ? beta_s[i] * m * As[i * DC_LDP + j] : 0.f;
    imgP[i * DC_LDP + j] = j <= i ? m * Ps[i * DC_LDP + j] : 0.f;
  }
  if (tid < DC_C) bg_s[tid] = beta_s[tid] * G_s[tid];
  if (tid == 0) imgP[DC_C] = G_s[DC_C - 1];     // (tokens behind the last one decay by nothing)
  __syncthreads();
  // ---- R: the two 16 x 16 blocks on the diagonal by forward substitution, a column a lane; then the block below
  if (tid < DC_C) {
    const int b = tid >> 4, j = tid & 15;
    float col[16];
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      float acc = i == j ? 1.f : 0.f;
#pragma unroll
      for (int m = 0; m < i; ++m) acc = fmaf(-As[(b * 16 + i) * DC_LDP + b * 16 + m], col[m], acc);
      col[i] = acc;
    }
#pragma unroll
    for (int i = 0; i < 16; ++i) Rs[(b * 16 + i) * DC_LDP + b * 16 + j] = col[i];
  } else if (tid >= 64) {
    // meanwhile the other waves put the queries and the keys into the image
    for (int i = (tid - 64) >> 3; i < DC_C; i += 24) {
      const float G = G_s[i];
      for (int d = 4 * (tid & 7); d < Dp; d += 32)
        *reinterpret_cast<ds_f32x4*>(imgQ + i * ld + d) = *reinterpret_cast<const ds_f32x4*>(Qs + i * ld + d) * G;
    }
    for (int e = tid - 64; e < DC_C * Dp; e += 192) {
      const int d = e >> 5, i = e & 31;
      imgK[d * DC_LDP + i] = Ks[i * ld + d] * Ms[(DC_C - 1) * DC_LDP + i];
    }
  }
  __syncthreads();
  {
    const int i = tid >> 4, j = tid & 15;
    float acc = 0.f;
#pragma unroll
    for (int m = 0; m < 16; ++m) acc = fmaf(As[(16 + i) * DC_LDP + m], Rs[m * DC_LDP + j], acc);
    Xs[i * DC_LDP + j] = acc;
    __syncthreads();
    acc = 0.f;
#pragma unroll
    for (int m = 0; m < 16; ++m) acc = fmaf(-Rs[(16 + i) * DC_LDP + 16 + m], Xs[m * DC_LDP + j], acc);
    Rs[(16 + i) * DC_LDP + j] = acc;
  }
  __syncthreads();
  // ---- W = R diag(beta G) K and U0 = R diag(beta) V, 16 columns a wave at a time
  const int wt = Dp >> 4, ut = (E + 15) >> 4;
  for (int ct = wave; ct < wt + ut; ct += 4) {
    const bool is_w = ct < wt;
    const int col = (is_w ? ct : ct - wt) * 16 + r16;
    const float* sc = is_w ? bg_s : beta_s;
    float b[8];       // the operand's rows 4 g4 + e, and 16 further on
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      const int j = (e >> 2) * 16 + 4 * g4 + (e & 3);
      if (is_w) b[e] = Ks[j * ld + col];
      else b[e] = (j < nt && col < E) ? to_float<T>(x[(long)(t0 + j) * ldx + v_off + (long)h * E + col]) : 0.f;
      b[e] *= sc[j];
    }
    ds_f32x4 lo = {0.f, 0.f, 0.f, 0.f}, hi = {0.f, 0.f, 0.f, 0.f};
    const ds_f32x4 a0 = *reinterpret_cast<const ds_f32x4*>(Rs + r16 * DC_LDP + 4 * g4);
    const ds_f32x4 a1 = *reinterpret_cast<const ds_f32x4*>(Rs + (16 + r16) * DC_LDP + 4 * g4);
    const ds_f32x4 a2 = *reinterpret_cast<const ds_f32x4*>(Rs + (16 + r16) * DC_LDP + 16 + 4 * g4);
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      lo = __builtin_amdgcn_mfma_f32_16x16x4f32(a0[e], b[e], lo, 0, 0, 0);
      hi = __builtin_amdgcn_mfma_f32_16x16x4f32(a1[e], b[e], hi, 0, 0, 0);
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) hi = __builtin_amdgcn_mfma_f32_16x16x4f32(a2[e], b[4 + e], hi, 0, 0, 0);
#pragma unroll
    for (int v = 0; v < 4; ++v) {
      const int i = 4 * g4 + v;
      if (is_w) {
        imgW[i * ld + col] = lo[v];
        imgW[(16 + i) * ld + col] = hi[v];
      } else if (col < E) {
        if (i < nt) out[(long)(t0 + i) * ldo + (long)h * E + col] = lo[v];
        if (16 + i < nt) out[(long)(t0 + 16 + i) * ldo + (long)h * E + col] = hi[v];
      }
    }
  }
}

// One workgroup per (request, head, EB value channels) walks the request's chunks of this step.  The state lies in
// LDS transposed, [value channel][d]; the next chunk's image travels from memory into registers while this
// one is multiplied.
template <int EB>
__global__ __launch_bounds__(256) void delta_chunk_kernel(
    const float* __restrict__ images, int n_head, int D, int E, const int* __restrict__ positions,
    float* __restrict__ state, long ld_state, const int* __restrict__ state_slots, const int* __restrict__ cu_q,
    float* __restrict__ out, long ldo) {
  constexpr int NJ = EB / 16;     // column tiles of the workgroup's value channels
  extern __shared__ __attribute__((aligned(16))) float dc_lds[];
  const int Dp = (D + 15) & ~15, ld = Dp + 4;
  const int img_floats = ds_image_floats(Dp), img4 = img_floats >> 2;
  float* Ws = dc_lds;                            // the image, as it lies in memory
  float* Qs = Ws + DC_C * ld;
  float* Kt = Qs + DC_C * ld;
  float* Ps = Kt + Dp * DC_LDP;
  float* St = dc_lds + img_floats;               // [EB][ld]
  float* Ut = St + EB * ld;                      // [EB][LDP]
  const int r = blockIdx.x, h = blockIdx.y, e0 = blockIdx.z * EB, tid = threadIdx.x;
  const int slot = state_slots[r];
  const int t_begin = cu_q[r], t_end = cu_q[r + 1];
  if (slot < 0 || t_end <= t_begin) return;     // a request of the padding
  const int wave = tid >> 6, lane = tid & 63, r16 = lane & 15, g4 = lane >> 4;
  float* st = state + (long)slot * ld_state + (long)h * D * E;
  const bool fresh = positions[t_begin] == 0;
  for (int i = tid; i < Dp * EB; i += 256) {
    const int d = i / EB, c = i - d * EB;
    St[c * ld + d] = (!fresh && d < D && e0 + c < E) ? st[(long)d * E + e0 + c] : 0.f;
  }
  // this wave's tile (oi, oj) of the chunk's [32, EB] updates and outputs; with 16 channels waves 0, 1 have the
  // updates and waves 2, 3 the outputs, with 32 a wave has both of its tile
  const int tile = EB == 32 ? wave : (wave & 1);
  const int oi = tile / NJ, oj = tile - oi * NJ;
  const bool has_u = EB == 32 || wave < 2, has_o = EB == 32 || wave >= 2;

  constexpr int IMG_PT = (2 * DC_C * (DC_DMAX + 4) + DC_DMAX * DC_LDP + DC_C * DC_LDP + 1023) / 1024;
  ds_f32x4 img_r[IMG_PT];
  float u0_r[4];
  const long first = (long)(t_begin / DC_C + r);
  const int n_chunks = (t_end - t_begin + DC_C - 1) / DC_C;
  auto fetch = [&](int ci) {
    const ds_f32x4* src = reinterpret_cast<const ds_f32x4*>(images + ((first + ci) * n_head + h) * img_floats);
#pragma unroll
    for (int u = 0; u < IMG_PT; ++u) {
      const int i = tid + u * 256;
      if (i < img4) img_r[u] = src[i];
    }
    if (has_u) {
#pragma unroll
      for (int v = 0; v < 4; ++v) {
        const int t = t_begin + ci * DC_C + oi * 16 + 4 * g4 + v, c = e0 + oj * 16 + r16;
        u0_r[v] = (t < t_end && c < E) ? out[(long)t * ldo + (long)h * E + c] : 0.f;
      }
    }
  };
  fetch(0);

  for (int ci = 0; ci < n_chunks; ++ci) {
    const int t0 = t_begin + ci * DC_C;
    const int nt = t_end - t0 < DC_C ? t_end - t0 : DC_C;
    __syncthreads();     // the chunk before is done with the image; S is whole
#pragma unroll
    for (int u = 0; u < IMG_PT; ++u) {
      const int i = tid + u * 256;
      if (i < img4) reinterpret_cast<ds_f32x4*>(dc_lds)[i] = img_r[u];
    }
    float u0[4];
#pragma unroll
    for (int v = 0; v < 4; ++v) u0[v] = u0_r[v];
    __syncthreads();
    if (ci + 1 < n_chunks) fetch(ci + 1);
    // ---- W S and diag(G) Q S
    ds_f32x4 aw = {0.f, 0.f, 0.f, 0.f}, aq = {0.f, 0.f, 0.f, 0.f};
    {
      const float* wrow = Ws + (oi * 16 + r16) * ld + 4 * g4;
      const float* qrow = Qs + (oi * 16 + r16) * ld + 4 * g4;
      const float* srow = St + (oj * 16 + r16) * ld + 4 * g4;
#pragma unroll 2
      for (int k0 = 0; k0 < Dp; k0 += 16) {
        const ds_f32x4 b = *reinterpret_cast<const ds_f32x4*>(srow + k0);
        if (has_u) {
          const ds_f32x4 a = *reinterpret_cast<const ds_f32x4*>(wrow + k0);
#pragma unroll
          for (int e = 0; e < 4; ++e) aw = __builtin_amdgcn_mfma_f32_16x16x4f32(a[e], b[e], aw, 0, 0, 0);
        }
        if (has_o) {
          const ds_f32x4 a = *reinterpret_cast<const ds_f32x4*>(qrow + k0);
#pragma unroll
          for (int e = 0; e < 4; ++e) aq = __builtin_amdgcn_mfma_f32_16x16x4f32(a[e], b[e], aq, 0, 0, 0);
        }
      }
    }
    if (has_u) {
      ds_f32x4 u;
#pragma unroll
      for (int v = 0; v < 4; ++v) u[v] = u0[v] - aw[v];
      *reinterpret_cast<ds_f32x4*>(Ut + (oj * 16 + r16) * DC_LDP + oi * 16 + 4 * g4) = u;
    }
    __syncthreads();     // U is whole, and every wave has read the old S
    // ---- O = diag(G) Q S + P U
    if (has_o) {
      for (int k0 = 0; k0 < (oi + 1) * 16; k0 += 16) {
        const ds_f32x4 a = *reinterpret_cast<const ds_f32x4*>(Ps + (oi * 16 + r16) * DC_LDP + k0 + 4 * g4);
        const ds_f32x4 b = *reinterpret_cast<const ds_f32x4*>(Ut + (oj * 16 + r16) * DC_LDP + k0 + 4 * g4);
#pragma unroll
        for (int e = 0; e < 4; ++e) aq = __builtin_amdgcn_mfma_f32_16x16x4f32(a[e], b[e], aq, 0, 0, 0);
      }
#pragma unroll
      for (int v = 0; v < 4; ++v) {
        const int i = oi * 16 + 4 * g4 + v, c = e0 + oj * 16 + r16;
        if (i < nt && c < E) out[(long)(t0 + i) * ldo + (long)h * E + c] = aq[v];
      }
    }
    // ---- S <- G_(n-1) S + K'^T U: the tiles (di, sj) of the [Dp, EB] state
    const float fall = Ps[DC_C];
    for (int t = wave; t < (Dp >> 4) * NJ; t += 4) {
      const int di = t / NJ, sj = t - di * NJ;
      ds_f32x4* mine = reinterpret_cast<ds_f32x4*>(St + (sj * 16 + r16) * ld + di * 16 + 4 * g4);   // rows d = 4 g4 + v of column r16
      ds_f32x4 acc = *mine;
#pragma unroll
      for (int v = 0; v < 4; ++v) acc[v] *= fall;
#pragma unroll
      for (int k0 = 0; k0 < DC_C; k0 += 16) {
        const ds_f32x4 a = *reinterpret_cast<const ds_f32x4*>(Kt + (di * 16 + r16) * DC_LDP + k0 + 4 * g4);
        const ds_f32x4 b = *reinterpret_cast<const ds_f32x4*>(Ut + (sj * 16 + r16) * DC_LDP + k0 + 4 * g4);
#pragma unroll
        for (int e = 0; e < 4; ++e) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a[e], b[e], acc, 0, 0, 0);
      }
      *mine = acc;
    }
  }
  __syncthreads();
  for (int i = tid; i < D * EB; i += 256) {
    const int d = i / EB, c = i - d * EB;
    if (e0 + c < E) st[(long)d * E + e0 + c] = St[c * ld + d];
  }
}

// float32 elements of `images` that mgpt_delta_state_chunked uses for a step of these sizes (0: it refuses them)
extern "C" long mgpt_delta_image_floats(int n_tokens, int n_req, int n_head, int head_dim) {
  if (n_tokens <= 0 || n_req <= 0 || n_head <= 0 || head_dim <= 0 || head_dim > DC_DMAX) return 0;
  return ((long)n_tokens / DC_C + n_req) * n_head * ds_image_floats((head_dim + 15) & ~15);
}

// The chunked form for steps with prompt portions: the arguments of mgpt_delta_state without the gate, and images,
// scratch of image_floats >= mgpt_delta_image_floats(...) elements.  out: float32 rows of all heads' values.  Head
// sizes up to 128 (value sizes up to 256); others are refused with MGPT_ERR_BAD_SHAPE and nothing launched.
extern "C" int mgpt_delta_state_chunked(const void* x, int dtype, long ldx, int q_off, int k_off, int v_off,
                                        const void* z, long ldz, int b_off, int a_off, int n_head, int n_group,
                                        int head_dim, int value_dim, float q_scale, const float* dt_bias,
                                        const float* a_log, float* state, long ld_state, const int* state_slots,
                                        const int* cu_q, int n_req, int n_tokens, const int* positions, float* images,
                                        long image_floats, float* out, long ldo, hipStream_t stream) {
  if (n_req == 0 || n_tokens == 0) return MGPT_OK;
  if (!x || !z || !dt_bias || !a_log || !state || !state_slots || !cu_q || !positions || !images || !out)
    return MGPT_ERR_NULL;
  if (!dtype_ok(dtype)) return MGPT_ERR_BAD_DTYPE;
  const int D = head_dim, E = value_dim;
  if (n_req < 0 || n_tokens < 0 || n_head <= 0 || n_group <= 0 || n_head % n_group || D <= 0 || E <= 0 || D > DC_DMAX ||
      E > DS_MAX || ld_state < (long)n_head * D * E || (((size_t)images) & 15) ||
      image_floats < mgpt_delta_image_floats(n_tokens, n_req, n_head, D))
    return MGPT_ERR_BAD_SHAPE;
  if (n_head > 65535) return MGPT_ERR_TOO_LARGE;
  const int Dp = (D + 15) & ~15, ld = Dp + 4;
  const int chunks = n_tokens / DC_C + n_req;
#define DC_ALLOW(kernel, bytes)                                                                              \
  {                                                                                                          \
    static int allowed = 0; /* more LDS than a kernel gets without asking */                                 \
    if (allowed < bytes) {                                                                                   \
      const hipError_t err = hipFuncSetAttribute(reinterpret_cast<const void*>(kernel),                      \
                                                 hipFuncAttributeMaxDynamicSharedMemorySize, bytes);        \
      if (err != hipSuccess) return (int)err;                                                                \
      allowed = bytes;                                                                                       \
    }                                                                                                        \
  }
  const size_t align = (size_t)x | (size_t)(ldx * (dtype == MGPT_F32 ? 4 : 2));
  const bool vec = !(D & 7) && !(align & 15) && !((q_off | k_off) & 7);
#define DC_PREPARE2(T, V)                                                                                                  \
  {                                                                                                                    \
    const int bytes = (int)sizeof(float) * (2 * DC_C * ld + 4 * DC_C * DC_LDP);                                       \
    DC_ALLOW((delta_prepare_kernel<T, V>), bytes)                                                                         \
    hipLaunchKernelGGL((delta_prepare_kernel<T, V>), dim3(chunks, n_head), dim3(256), bytes, stream, (const T*)x, ldx,    \
                       q_off, k_off, v_off, (const T*)z, ldz, b_off, a_off, n_head, n_head / n_group, D, E, q_scale,   \
                       dt_bias, a_log, cu_q, n_req, images, out, ldo);                                                 \
  }
#define DC_PREPARE(T)                                        \
  {                                                          \
    if (vec) DC_PREPARE2(T, true) else DC_PREPARE2(T, false) \
  }
  if (dtype == MGPT_F32) DC_PREPARE(float) else DC_PREPARE(bf16_t)
#define DC_WALK(EB)                                                                                              \
  {                                                                                                              \
    const int bytes = (int)sizeof(float) * (ds_image_floats(Dp) + EB * ld + EB * DC_LDP);                       \
    DC_ALLOW((delta_chunk_kernel<EB>), bytes)                                                                    \
    hipLaunchKernelGGL((delta_chunk_kernel<EB>), dim3(n_req, n_head, (E + EB - 1) / EB), dim3(256), bytes, stream, \
                       images, n_head, D, E, positions, state, ld_state, state_slots, cu_q, out, ldo);           \
  }
  // 32 value channels a workgroup; 16 where that many workgroups would leave compute units idle
  if ((long)n_req * n_head * ((E + 31) / 32) >= 256) DC_WALK(32) else DC_WALK(16)
#undef DC_WALK
#undef DC_PREPARE
#undef DC_PREPARE2
#undef DC_ALLOW
  return mgpt_last_error();
}
