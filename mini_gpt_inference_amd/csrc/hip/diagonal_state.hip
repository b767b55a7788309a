// A linear recurrence with a float32 state of one number per channel, whose decay and input gate come from the token:
//
//   a = exp(decay[c] * sigmoid(gr + r_bias)),   i = sigmoid(gi + i_bias)
//   S <- a S + i u sqrt(1 - a^2);   out = S * gelu_tanh(y)      (without y: S)
//
// decay[c] <= 0 is a number per channel.  The two gates' logits lie block by block in the rows of g: for the channels of
// block b (`block` of them) gr at columns 2 b block .., gi at (2 b + 1) block ...  S is zero before a request's first
// token and comes from, and goes back to, the request's slot of a pool; from the loaded numbers on everything is float32.
// That root is taken as sqrt(-expm1(2 log a)), which is exact where a is nearly 1.
#include "common.h"
#include "dtype_io.h"
#include "launchers.h"

#define DG_C 32      // tokens a chunk

struct DgStep {
  float a, x;     // the state becomes a * S + x
};

// 1 - a^2 for a = exp(t / 2), t <= 0: near t = 0 by the series of 1 - exp(t) (seven terms, below 2^-25 relative up to
// 1/4), elsewhere from a
__device__ __forceinline__ float dg_one_minus_square(float a, float t) {
  float p = 1.0f / 5040.0f;
  p = fmaf(p, t, 1.0f / 720.0f);
  p = fmaf(p, t, 1.0f / 120.0f);
  p = fmaf(p, t, 1.0f / 24.0f);
  p = fmaf(p, t, 1.0f / 6.0f);
  p = fmaf(p, t, 0.5f);
  p = fmaf(p, t, 1.0f);
  return t > -0.25f ? -t * p : fmaf(-a, a, 1.0f);
}

// FAST: the hardware's exp2, reciprocal and square root (a few ulp of float32), for rows in bfloat16
template <bool FAST>
__device__ __forceinline__ DgStep dg_step(float u, float gr, float gi, float decay) {
  DgStep s;
  if (FAST) {
    const float k = -1.4426950408889634f;
    const float log_a = decay * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(k * gr));
    s.a = __builtin_amdgcn_exp2f(log_a * 1.4426950408889634f);
    s.x = __builtin_amdgcn_sqrtf(dg_one_minus_square(s.a, 2.0f * log_a)) * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(k * gi)) * u;
  } else {
    const float log_a = decay / (1.0f + expf(-gr));
    s.a = expf(log_a);
    s.x = sqrtf(-expm1f(2.0f * log_a)) / (1.0f + expf(-gi)) * u;
  }
  return s;
}

template <bool FAST> __device__ __forceinline__ float dg_gelu(float v) { return FAST ? gelu_tanh_fast(v) : gelu_tanh(v); }

// Single tokens: a thread a (request, channel), the request's tokens in order.
template <typename UT, typename GT, typename YT, typename OT>
__global__ __launch_bounds__(256) void diagonal_state_kernel(
    const UT* __restrict__ u, long ldu, const GT* __restrict__ g, long ldg, const float* __restrict__ r_bias,
    const float* __restrict__ i_bias, const float* __restrict__ decay, int block, const YT* __restrict__ y, long ldy, int y_off,
    float* __restrict__ state, long ld_state, const int* __restrict__ state_slots, const int* __restrict__ cu_q,
    const int* __restrict__ positions, int C, OT* __restrict__ out, long ldo) {
  const int r = blockIdx.x, c = blockIdx.y * 256 + threadIdx.x;
  const int slot = state_slots[r], t0 = cu_q[r], t1 = cu_q[r + 1];
  if (slot < 0 || t1 <= t0 || c >= C) return;     // a request of the padding
  const int gc = 2 * (c / block) * block + c % block;
  const float rb = r_bias[c], ib = i_bias[c], dc = decay[c];
  float* const st = state + (long)slot * ld_state + c;
  float S = positions[t0] == 0 ? 0.f : *st;
  constexpr bool FAST = sizeof(UT) == 2;
  for (int t = t0; t < t1; ++t) {
    const DgStep s = dg_step<FAST>(to_float<UT>(u[(long)t * ldu + c]), to_float<GT>(g[(long)t * ldg + gc]) + rb,
                             to_float<GT>(g[(long)t * ldg + gc + block]) + ib, dc);
    S = fmaf(s.a, S, s.x);
    const float v = y ? S * dg_gelu<FAST>(to_float<YT>(y[(long)t * ldy + y_off + c])) : S;
    out[(long)t * ldo + c] = from_float<OT>(v);
  }
  *st = S;
}

// Prompt portions: chunks of DG_C tokens counted from the portion's start, side by side.  The chunks of request r have the
// numbers cu_q[r] / DG_C + r and following.  A first pass leaves per chunk and channel what the chunk does to a state,
// S -> A S + X (the first chunk, whose state is known, leaves that state and its own end); the second puts the
// chunks before together, in order, and goes through the tokens again with the state that comes out.
// scratch: [3][chunks][C]: A, X (a first chunk's: its end), a first chunk's state at its start.
template <typename UT, typename GT, typename YT, typename OT, bool LAST>
__global__ __launch_bounds__(256) void diagonal_chunk_kernel(
    const UT* __restrict__ u, long ldu, const GT* __restrict__ g, long ldg, const float* __restrict__ r_bias,
    const float* __restrict__ i_bias, const float* __restrict__ decay, int block, const YT* __restrict__ y, long ldy, int y_off,
    float* __restrict__ state, long ld_state, const int* __restrict__ state_slots, const int* __restrict__ cu_q,
    const int* __restrict__ positions, int n_req, int C, float* __restrict__ scratch, OT* __restrict__ out, long ldo) {
  const int chunk = blockIdx.x, c = blockIdx.y * 256 + threadIdx.x;
  // the request whose chunks this number belongs to: its first number rises with r
  int r = -1;
  for (int base = 0; base < n_req; base += 256) {
    const int s = base + (int)threadIdx.x;
    r += __syncthreads_count(s < n_req && cu_q[s < n_req ? s : 0] / DG_C + s <= chunk);
  }
  if (r < 0) return;
  const int first = cu_q[r] / DG_C + r;
  const int t0 = cu_q[r] + (chunk - first) * DG_C, end = cu_q[r + 1], slot = state_slots[r];
  if (t0 >= end || slot < 0 || c >= C) return;      // a number without a chunk, a request of the padding
  const int t1 = t0 + DG_C < end ? t0 + DG_C : end;
  const long plane = (long)gridDim.x * C;
  float* const mine = scratch + (long)chunk * C + c;
  const int gc = 2 * (c / block) * block + c % block;
  const float rb = r_bias[c], ib = i_bias[c], dc = decay[c];
  float* const st = state + (long)slot * ld_state + c;
  constexpr bool FAST = sizeof(UT) == 2;
  float S = 0.f, A = 1.f;
  if (!LAST) {
    if (chunk == first) {
      if (positions[t0] != 0) S = *st;
      mine[2 * plane] = S;
    }
  } else if (chunk == first) {
    S = mine[2 * plane];
  } else {
    const float* before = scratch + (long)first * C + c;
    S = before[plane];
#pragma unroll 8
    for (int k = first + 1; k < chunk; ++k) {
      before += C;
      S = fmaf(before[0], S, before[plane]);
    }
  }
#pragma unroll 8
  for (int t = t0; t < t1; ++t) {
    const DgStep s = dg_step<FAST>(to_float<UT>(u[(long)t * ldu + c]), to_float<GT>(g[(long)t * ldg + gc]) + rb,
                             to_float<GT>(g[(long)t * ldg + gc + block]) + ib, dc);
    S = fmaf(s.a, S, s.x);
    if (!LAST) {
      A *= s.a;
    } else {
      const float v = y ? S * dg_gelu<FAST>(to_float<YT>(y[(long)t * ldy + y_off + c])) : S;
      out[(long)t * ldo + c] = from_float<OT>(v);
    }
  }
  if (!LAST) {
    mine[0] = A;
    mine[plane] = S;
  } else if (t1 == end) {
    *st = S;      // (every first chunk's state was read by the pass before)
  }
}

// u: rows of `channels` columns; g: rows of 2 * channels columns; y: rows whose channels start at y_off, or null; state:
// rows of ld_state floats of which the first `channels` are used; scratch: at least 3 * (n_tokens / 32 + n_req) *
// channels floats for steps in which a request brings several tokens (null: every request brings one).
// Types: g float32 or u's type; y and out u's type, or out float32.
extern "C" int mgpt_diagonal_state(const void* u, int u_dtype, long ldu, const void* g, int g_dtype, long ldg,
                                   const float* r_bias, const float* i_bias, const float* decay, int block, const void* y,
                                   int y_dtype, long ldy, int y_off, float* state, long ld_state, const int* state_slots,
                                   const int* cu_q, const int* positions, int n_req, int n_tokens, int channels,
                                   float* scratch, long scratch_floats, void* out, int out_dtype, long ldo,
                                   hipStream_t stream) {
  if (n_tokens == 0 || n_req == 0) return MGPT_OK;
  if (!u || !g || !r_bias || !i_bias || !decay || !state || !state_slots || !cu_q || !positions || !out) return MGPT_ERR_NULL;
  if (!dtype_ok(u_dtype) || !dtype_ok(g_dtype) || !dtype_ok(out_dtype)) return MGPT_ERR_BAD_DTYPE;
  if ((y && y_dtype != u_dtype) || out_dtype != u_dtype || (g_dtype != MGPT_F32 && g_dtype != u_dtype)) return MGPT_ERR_BAD_DTYPE;
  if (n_tokens < 0 || n_req < 0 || channels <= 0 || block <= 0 || channels % block || ldu < channels || ldg < 2L * channels ||
      ldo < channels || ld_state < channels || (y && (y_off < 0 || ldy < y_off + (long)channels)))
    return MGPT_ERR_BAD_SHAPE;
  const int cb = (channels + 255) / 256;
  if (cb > 65535) return MGPT_ERR_TOO_LARGE;
  const int chunks = n_tokens / DG_C + n_req;
  if (scratch && scratch_floats < 3L * chunks * channels) return MGPT_ERR_BAD_SHAPE;
#define DG_ARGS(UT, GT) (const UT*)u, ldu, (const GT*)g, ldg, r_bias, i_bias, decay, block, (const UT*)y, ldy, y_off, state, \
                        ld_state, state_slots, cu_q, positions
#define DG_LAUNCH(UT, GT)                                                                                              \
  {                                                                                                                    \
    if (!scratch)                                                                                                      \
      hipLaunchKernelGGL((diagonal_state_kernel<UT, GT, UT, UT>), dim3(n_req, cb), dim3(256), 0, stream, DG_ARGS(UT, GT), \
                         channels, (UT*)out, ldo);                                                                     \
    else {                                                                                                             \
      hipLaunchKernelGGL((diagonal_chunk_kernel<UT, GT, UT, UT, false>), dim3(chunks, cb), dim3(256), 0, stream,       \
                         DG_ARGS(UT, GT), n_req, channels, scratch, (UT*)out, ldo);                                    \
      hipLaunchKernelGGL((diagonal_chunk_kernel<UT, GT, UT, UT, true>), dim3(chunks, cb), dim3(256), 0, stream,        \
                         DG_ARGS(UT, GT), n_req, channels, scratch, (UT*)out, ldo);                                    \
    }                                                                                                                  \
  }
  if (u_dtype == MGPT_F32) DG_LAUNCH(float, float)
  else if (g_dtype == MGPT_F32) DG_LAUNCH(bf16_t, float)
  else DG_LAUNCH(bf16_t, bf16_t)
#undef DG_LAUNCH
#undef DG_ARGS
  return mgpt_last_error();
}

// ---------------------------------------------------------------------------------------------
// bfloat16 rows, blocks of a multiple of 16 channels: the gates' products on the matrix cores inside the recurrence's
// kernels, their sums (float32) never leaving the registers.
typedef __attribute__((__vector_size__(8 * sizeof(short)))) short dg_bf16x8_t;
typedef __attribute__((__vector_size__(4 * sizeof(float)))) float dg_f32x4_t;

#define DF_C 64            // tokens a chunk
#define DF_CH 128          // channels a workgroup at most, 16 a wave
#define DF_MAX_TAPS 9
#define DF_MAX_BLOCK 512

struct DfArgs {
  const bf16_t* z;         // rows with the branch in front of the convolution (columns 0 ..) and y (columns y_off ..)
  long ldz;
  int y_off;
  const float* conv_w;     // [taps][channels]
  const float* conv_b;     // [channels]
  int taps;
  const bf16_t* w;         // [channels / 16][2][block / 32, rounded up][64][8]: see below
  const float *r_bias, *i_bias, *decay;
  int block, channels;
  float* state;            // rows of ld_state floats: [channels] the state
  float* kept;             // the same rows' [taps - 1][channels] convolution inputs
  long ld_state;
  const int *state_slots, *cu_q, *positions;
  int n_req;
  float* scratch;          // [2][rows][channels]: what a chunk's tokens up to a row do to a state, S -> A S + X
  long plane;
  const bf16_t* u;         // single tokens: the convolution's output, [rows][channels]
  bf16_t* out;
  long ldo;
};

// value of lane l - 16 * D (lanes below get their own)
__device__ __forceinline__ float df_up(float v, int d) { return __shfl_up(v, 16 * d, 64); }

struct DfChunk {
  int start, end, slot, t0, n_valid;      // the request's rows and slot; the chunk's first row and number of rows
  int first;                              // the number of the request's first chunk
};

// the chunk of a number (as for diagonal_chunk_kernel, of 64 tokens); false: a number without a chunk.  Every thread of
// the workgroup calls it.
__device__ __forceinline__ bool df_find(const DfArgs& p, int chunk, DfChunk& out) {
  int r = -1;
  for (int base = 0; base < p.n_req; base += blockDim.x) {
    const int s = base + (int)threadIdx.x;
    r += __syncthreads_count(s < p.n_req && p.cu_q[s < p.n_req ? s : 0] / DF_C + s <= chunk);
  }
  if (r < 0) return false;
  out.start = p.cu_q[r];
  out.end = p.cu_q[r + 1];
  out.slot = p.state_slots[r];
  out.first = out.start / DF_C + r;
  out.t0 = out.start + (chunk - out.first) * DF_C;
  out.n_valid = out.end - out.t0 < DF_C ? out.end - out.t0 : DF_C;
  return out.t0 < out.end && out.slot >= 0;
}

// The gates' matrices come in the order in which the waves take them: for every 16 channels first r, then i, and of
// each, 32 inner channels at a time, lane (g, c)'s eight values: channel c of the sixteen, inner channels 8 g .. 8 g + 7
// (zeros behind the block's end).  A wave's load is then 1 KB in a row.
//
// First pass.  A workgroup takes a chunk of 64 tokens and up to 128 channels of one block, a wave 16 of them.  It makes
// the convolution's rows of the chunk for the whole block (the products need them all) in LDS and multiplies the gates
// out, tokens along the rows of the result: lane (g, c) of a wave then holds tokens 4 g .. 4 g + 3 of each of four
// 16-token tiles of its channel c, goes through its four, and the four lanes of a channel and the tiles are put together
// by (a', x') after (a, x) = (a a', a' x + x').  Stored is, per token, what the chunk's tokens up to it do to the state
// at the chunk's start; a request's first chunk starts from the request's state, which is known.
__global__ __launch_bounds__(512) void diagonal_gates_kernel(DfArgs p) {
  extern __shared__ __align__(16) bf16_t df_lds[];     // [64][block + 8]
  const int tid = threadIdx.x, threads = blockDim.x, lane = tid & 63, wave = tid >> 6;
  DfChunk ck;
  if (!df_find(p, blockIdx.x, ck)) return;
  const int block = p.block, C = p.channels;
  const int groups = (block + DF_CH - 1) / DF_CH;
  const int b = blockIdx.y / groups, own = (blockIdx.y - b * groups) * DF_CH;    // own: first channel of the workgroup in its block
  const int base_c = b * block;
  const int ld_u = block + 8, pieces = block / 8;
  bf16_t* const u_s = df_lds;
  const dg_bf16x8_t zero8 = {0, 0, 0, 0, 0, 0, 0, 0};
  {
    const int H = p.taps - 1;
    const bool inside = ck.t0 - H >= ck.start;         // no tap reaches back before this step's tokens
    const int pos0 = inside ? 0 : p.positions[ck.start];
    for (int idx = tid; idx < DF_C * pieces; idx += threads) {
      const int i = idx / pieces, c = (idx - i * pieces) * 8;
      dg_bf16x8_t o = zero8;
      if (i < ck.n_valid) {
        float acc[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) acc[e] = p.conv_b[base_c + c + e];
        const bf16_t* src = p.z + (long)(ck.t0 + i - H) * p.ldz + base_c + c;
        const float* w = p.conv_w + base_c + c;
        if (inside) {
#pragma unroll 4
          for (int j = 0; j < p.taps; ++j) {
            const dg_bf16x8_t v = *reinterpret_cast<const dg_bf16x8_t*>(src + (long)j * p.ldz);
#pragma unroll
            for (int e = 0; e < 8; ++e) acc[e] = fmaf(w[(long)j * C + e], bf16_to_float((bf16_t)v[e]), acc[e]);
          }
        } else {
          for (int j = 0; j < p.taps; ++j) {
            const int back = ck.start - (ck.t0 + i - H + j);      // > 0: an input of an earlier step
            if (back <= 0) {
              const dg_bf16x8_t v = *reinterpret_cast<const dg_bf16x8_t*>(src + (long)j * p.ldz);
#pragma unroll
              for (int e = 0; e < 8; ++e) acc[e] = fmaf(w[(long)j * C + e], bf16_to_float((bf16_t)v[e]), acc[e]);
            } else if (pos0 - back >= 0) {
              const float* k = p.kept + (long)ck.slot * p.ld_state + (long)(H - back) * C + base_c + c;
#pragma unroll
              for (int e = 0; e < 8; ++e) acc[e] = fmaf(w[(long)j * C + e], k[e], acc[e]);
            }
          }
        }
#pragma unroll
        for (int e = 0; e < 8; ++e) o[e] = (short)float_to_bf16(acc[e]);
      }
      *reinterpret_cast<dg_bf16x8_t*>(u_s + i * ld_u + c) = o;
    }
  }
  __syncthreads();

  const int li = lane & 15, g = lane >> 4;
  const int ch = own + wave * 16 + li;                 // this lane's channel in the block
  if (own + wave * 16 >= block) return;                // (the whole wave: blocks are multiples of 16)
  dg_f32x4_t ar[4], ai[4];
#pragma unroll
  for (int t = 0; t < 4; ++t) ar[t] = ai[t] = dg_f32x4_t{0.f, 0.f, 0.f, 0.f};
  const int k_steps = (block + 31) / 32;
  const bf16_t* wr = p.w + ((long)(base_c + own) / 16 + wave) * 2 * k_steps * 512 + lane * 8;
  const bf16_t* wi = wr + k_steps * 512;
#pragma unroll 4
  for (int ks = 0; ks < k_steps; ++ks) {
    const int k = ks * 32 + g * 8;
    const bool k_ok = k < block;
    const dg_bf16x8_t fr = *reinterpret_cast<const dg_bf16x8_t*>(wr + ks * 512);
    const dg_bf16x8_t fi = *reinterpret_cast<const dg_bf16x8_t*>(wi + ks * 512);
#pragma unroll
    for (int t = 0; t < 4; ++t) {
      const dg_bf16x8_t fu = k_ok ? *reinterpret_cast<const dg_bf16x8_t*>(u_s + (t * 16 + li) * ld_u + k) : zero8;
      ar[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fu, fr, ar[t], 0, 0, 0);
      ai[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fu, fi, ai[t], 0, 0, 0);
    }
  }
  const int c = base_c + ch;
  const float rb = p.r_bias[c], ib = p.i_bias[c], dc = p.decay[c];
  float S = 0.f, A = 1.f;                              // of the chunk's tokens before the tile
  if ((int)blockIdx.x == ck.first && p.positions[ck.t0] != 0) S = p.state[(long)ck.slot * p.ld_state + c];
  float* const at = p.scratch + (long)(ck.t0 + g * 4) * C + c;
#pragma unroll
  for (int t = 0; t < 4; ++t) {
    float la = 1.f, lx = 0.f;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int row = t * 16 + g * 4 + i;
      DgStep s = dg_step<true>(bf16_to_float(u_s[row * ld_u + ch]), ar[t][i] + rb, ai[t][i] + ib, dc);
      if (row >= ck.n_valid) {      // behind the request's last token: the state stays
        s.a = 1.f;
        s.x = 0.f;
      }
      lx = fmaf(s.a, lx, s.x);
      la *= s.a;
      ar[t][i] = la;
      ai[t][i] = lx;
    }
#pragma unroll
    for (int d = 1; d <= 2; ++d) {
      const float pa = df_up(la, d), px = df_up(lx, d);
      if (g >= d) {
        lx = fmaf(la, px, lx);
        la *= pa;
      }
    }
    const float ea = df_up(la, 1), ex = df_up(lx, 1);
    // up to this lane's tokens: the chunk's tiles before, then the lanes before in this tile
    const float ba = g ? A * ea : A, bx = g ? fmaf(ea, S, ex) : S;
    const float ta = __shfl(la, 48 + li, 64), tx = __shfl(lx, 48 + li, 64);
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (t * 16 + g * 4 + i < ck.n_valid) {
        at[(long)(t * 16 + i) * C] = ar[t][i] * ba;
        at[p.plane + (long)(t * 16 + i) * C] = fmaf(ar[t][i], bx, ai[t][i]);
      }
    S = fmaf(ta, S, tx);
    A *= ta;
  }
}

#define DF_T 8             // tokens a thread of the second pass

// Second pass: the state at the chunk's start from the ends of the chunks before, in order, then every token's state and
// output.  A workgroup takes 32 tokens of a chunk and 256 channels, a thread eight tokens of four channels.
__global__ __launch_bounds__(256) void diagonal_output_kernel(DfArgs p) {
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  DfChunk ck;
  if (!df_find(p, blockIdx.x, ck)) return;
  const int C = p.channels, c = blockIdx.y * 256 + lane * 4;
  if (c >= C) return;                                  // (four channels at a time: they are a multiple of 16)
  const int i0 = (blockIdx.z * 4 + wave) * DF_T;       // the thread's first token in the chunk
  if (i0 >= ck.n_valid) return;
  const int n = ck.n_valid - i0 < DF_T ? ck.n_valid - i0 : DF_T;
  const float* src = p.scratch + (long)(ck.t0 + i0) * C + c;
  float4 a[DF_T], x[DF_T];
  uint2 y[DF_T];
#pragma unroll
  for (int i = 0; i < DF_T; ++i) {
    const int k = i < n ? i : n - 1;
    a[i] = *reinterpret_cast<const float4*>(src + (long)k * C);
    x[i] = *reinterpret_cast<const float4*>(src + p.plane + (long)k * C);
    y[i] = *reinterpret_cast<const uint2*>(p.z + (long)(ck.t0 + i0 + k) * p.ldz + p.y_off + c);
  }
  float4 S = make_float4(0.f, 0.f, 0.f, 0.f);
  // the ends of the request's chunks before this one: their last rows
  const float* end_row = p.scratch + (long)(ck.start + DF_C - 1) * C + c;
#pragma unroll 4
  for (int k = ck.first; k < (int)blockIdx.x; ++k) {
    const float4 ea = *reinterpret_cast<const float4*>(end_row), ex = *reinterpret_cast<const float4*>(end_row + p.plane);
    S.x = fmaf(ea.x, S.x, ex.x);
    S.y = fmaf(ea.y, S.y, ex.y);
    S.z = fmaf(ea.z, S.z, ex.z);
    S.w = fmaf(ea.w, S.w, ex.w);
    end_row += (long)DF_C * C;
  }
  float4 v;
#pragma unroll
  for (int i = 0; i < DF_T; ++i) {
    if (i >= n) break;
    v = make_float4(fmaf(a[i].x, S.x, x[i].x), fmaf(a[i].y, S.y, x[i].y), fmaf(a[i].z, S.z, x[i].z), fmaf(a[i].w, S.w, x[i].w));
    uint2 o;
    o.x = pack_bf16x2(v.x * dg_gelu<true>(__uint_as_float(y[i].x << 16)), v.y * dg_gelu<true>(__uint_as_float(y[i].x & 0xffff0000u)));
    o.y = pack_bf16x2(v.z * dg_gelu<true>(__uint_as_float(y[i].y << 16)), v.w * dg_gelu<true>(__uint_as_float(y[i].y & 0xffff0000u)));
    *reinterpret_cast<uint2*>(p.out + (long)(ck.t0 + i0 + i) * p.ldo + c) = o;
  }
  if (ck.t0 + i0 + n != ck.end) return;
  // the request's last token: its state, and the convolution's last inputs (the pass before was the last to read either)
  float* st = p.state + (long)ck.slot * p.ld_state + c;
  st[0] = v.x;
  st[1] = v.y;
  st[2] = v.z;
  st[3] = v.w;
  const int H = p.taps - 1, len = ck.end - ck.start;
  float* kp = p.kept + (long)ck.slot * p.ld_state + c;
  for (int i = 0; i < H; ++i) {      // (the rows move up: row i is written after it, and before any later one, is read)
    const int t = ck.end - H + i;
#pragma unroll
    for (int e = 0; e < 4; ++e)
      kp[(long)i * C + e] = t >= ck.start ? bf16_to_float(p.z[(long)t * p.ldz + c + e]) : kp[(long)(i + len) * C + e];
  }
}

// Single tokens (token n is request n): a workgroup takes 16 tokens and 16 channels of a block, the inner size dealt out
// to four waves; then a thread a (token, channel).  u: the convolution's output.
__global__ __launch_bounds__(256) void diagonal_step_kernel(DfArgs p, int n_tokens) {
  __shared__ dg_f32x4_t part[4][2][64];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, li = lane & 15, g = lane >> 4;
  const int block = p.block, C = p.channels;
  const int c0 = blockIdx.x * 16, b = c0 / block, n0 = blockIdx.y * 16;
  // what the thread's own element needs: asked for ahead of the products
  const int row = n0 + (tid >> 4), c = c0 + (tid & 15);
  const bool have = row < n_tokens && row < p.n_req;
  const int slot = have ? p.state_slots[row] : -1;
  const bool live = have && slot >= 0 && p.cu_q[row + 1] > p.cu_q[row];
  const float uv = live ? bf16_to_float(p.u[(long)row * C + c]) : 0.f;
  const float yv = live ? bf16_to_float(p.z[(long)row * p.ldz + p.y_off + c]) : 0.f;
  float S = live && p.positions[row] != 0 ? p.state[(long)slot * p.ld_state + c] : 0.f;
  const float rb = p.r_bias[c], ib = p.i_bias[c], dc = p.decay[c];
  const dg_bf16x8_t zero8 = {0, 0, 0, 0, 0, 0, 0, 0};
  dg_f32x4_t ar = {0.f, 0.f, 0.f, 0.f}, ai = {0.f, 0.f, 0.f, 0.f};
  const int k_steps = (block + 31) / 32;
  const bf16_t* wr = p.w + (long)blockIdx.x * 2 * k_steps * 512 + lane * 8;
  const bf16_t* wi = wr + k_steps * 512;
  const int ur = n0 + li;
  const bf16_t* up = p.u + (long)(ur < n_tokens ? ur : 0) * C + b * block;
#pragma unroll 2
  for (int ks = wave; ks < k_steps; ks += 4) {
    const int k = ks * 32 + g * 8;
    const bool k_ok = k < block;
    const dg_bf16x8_t fr = *reinterpret_cast<const dg_bf16x8_t*>(wr + ks * 512);
    const dg_bf16x8_t fi = *reinterpret_cast<const dg_bf16x8_t*>(wi + ks * 512);
    const dg_bf16x8_t fu = k_ok && ur < n_tokens ? *reinterpret_cast<const dg_bf16x8_t*>(up + k) : zero8;
    ar = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fu, fr, ar, 0, 0, 0);
    ai = __builtin_amdgcn_mfma_f32_16x16x32_bf16(fu, fi, ai, 0, 0, 0);
  }
  part[wave][0][lane] = ar;
  part[wave][1][lane] = ai;
  __syncthreads();
  if (!live) return;
  const int rr = tid >> 4, at = (rr >> 2) * 16 + (tid & 15), i = rr & 3;
  const float gr = (part[0][0][at][i] + part[1][0][at][i]) + (part[2][0][at][i] + part[3][0][at][i]);
  const float gi = (part[0][1][at][i] + part[1][1][at][i]) + (part[2][1][at][i] + part[3][1][at][i]);
  const DgStep s = dg_step<true>(uv, gr + rb, gi + ib, dc);
  S = fmaf(s.a, S, s.x);
  p.state[(long)slot * p.ld_state + c] = S;
  p.out[(long)row * p.ldo + c] = float_to_bf16(S * dg_gelu<true>(yv));
}

// z: bfloat16 rows, the branch in front of the convolution at column 0 and y at y_off; conv_w float32 [taps][channels];
// w bfloat16 in the kernels' order; state: rows of ld_state floats, the state at column 0 and the convolution's last
// inputs at column `channels`.  With scratch (2 * n_tokens * channels floats) a step in which requests bring several
// tokens: convolution, gates, recurrence, state and inputs brought up to date.  Without one a step of single tokens with
// the convolution's output in u (dense rows of `channels`; its inputs kept by the caller).  Refuses (MGPT_ERR_BAD_SHAPE)
// blocks that are no multiple of 16 or larger than DF_MAX_BLOCK and rows that do not take 16-byte loads.
extern "C" int mgpt_diagonal_state_fused(const void* z, long ldz, int y_off, const float* conv_w, const float* conv_b, int taps,
                                         const void* w, const float* r_bias, const float* i_bias, const float* decay, int block,
                                         int channels, float* state, long ld_state, const int* state_slots, const int* cu_q,
                                         const int* positions, int n_req, int n_tokens, float* scratch, long scratch_floats,
                                         const void* u, void* out, long ldo, hipStream_t stream) {
  if (n_tokens == 0 || n_req == 0) return MGPT_OK;
  if (!z || !w || !r_bias || !i_bias || !decay || !state || !state_slots || !cu_q || !positions || !out) return MGPT_ERR_NULL;
  if (scratch ? (!conv_w || !conv_b) : !u) return MGPT_ERR_NULL;
  if (n_tokens < 0 || n_req < 0 || channels <= 0 || block <= 0 || block > DF_MAX_BLOCK || (block & 15) || channels % block ||
      taps < 1 || taps > DF_MAX_TAPS || ldz < channels || y_off < 0 || ldz < y_off + (long)channels || ldo < channels ||
      ld_state < (long)taps * channels || (ldz & 7) || (y_off & 7) || (ldo & 7) ||
      (((size_t)z | (size_t)w | (size_t)u | (size_t)out | (size_t)scratch) & 15))
    return MGPT_ERR_BAD_SHAPE;
  const long plane = (long)n_tokens * channels;
  DfArgs p = {(const bf16_t*)z, ldz, y_off, conv_w, conv_b, taps, (const bf16_t*)w, r_bias, i_bias, decay, block, channels,
              state, state + channels, ld_state, state_slots, cu_q, positions, n_req, scratch, plane, (const bf16_t*)u, (bf16_t*)out, ldo};
  if (!scratch) {
    if (n_tokens > n_req) return MGPT_ERR_BAD_SHAPE;      // (a token a request)
    const int tiles = (n_tokens + 15) / 16;
    if (tiles > 65535) return MGPT_ERR_TOO_LARGE;
    hipLaunchKernelGGL(diagonal_step_kernel, dim3(channels / 16, tiles), dim3(256), 0, stream, p, n_tokens);
    return mgpt_last_error();
  }
  if (scratch_floats < 2 * plane) return MGPT_ERR_BAD_SHAPE;
  const int chunks = n_tokens / DF_C + n_req;
  const int groups = (channels / block) * ((block + DF_CH - 1) / DF_CH);
  if (groups > 65535) return MGPT_ERR_TOO_LARGE;
  const int bytes = DF_C * (block + 8) * (int)sizeof(bf16_t);
  static bool allowed = false;
  if (!allowed) {
    const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(diagonal_gates_kernel),
                                             hipFuncAttributeMaxDynamicSharedMemorySize, DF_C * (DF_MAX_BLOCK + 8) * 2);
    if (e != hipSuccess) return (int)e;
    allowed = true;
  }
  const int threads = (block < DF_CH ? block : DF_CH) / 16 * 64;
  hipLaunchKernelGGL(diagonal_gates_kernel, dim3(chunks, groups), dim3(threads), bytes, stream, p);
  hipLaunchKernelGGL(diagonal_output_kernel, dim3(chunks, (channels + 255) / 256, DF_C / (4 * DF_T)), dim3(256), 0, stream, p);
  return mgpt_last_error();
}
