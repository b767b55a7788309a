// A linear recurrence with a float32 state of one number per channel, whose decay and input gate come from the token:
//
//   r = sigmoid(gr + r_bias), i = sigmoid(gi + i_bias), log a = decay[c] * r, a = exp(log a)
//   S_t = a S_(t-1) + sqrt(1 - a^2) i u_t;   out_t = S_t * gelu_tanh(y_t)      (without y: S_t)
//
// decay[c] <= 0 is a number per channel.  The two gates' logits lie block by block in the rows of g: for the channels of
// block b (`block` of them) gr at columns 2 b block .., gi at (2 b + 1) block ...  S is zero before a request's first
// token and comes from, and goes back to, the request's slot of a pool; from the loaded numbers on everything is float32.
// sqrt(1 - a^2) is taken as sqrt(-expm1(2 log a)), which is exact where a is nearly 1.
#include "common.h"
#include "dtype_io.h"
#include "launchers.h"

#define DG_C 32      // tokens a chunk

__device__ __forceinline__ float dg_sigmoid(float v) { return 1.0f / (1.0f + expf(-v)); }

struct DgStep {
  float a, log_a, x;     // the state becomes a * S + x
};

__device__ __forceinline__ DgStep dg_step(float u, float gr, float gi, float decay) {
  DgStep s;
  s.log_a = decay * dg_sigmoid(gr);
  s.a = expf(s.log_a);
  s.x = sqrtf(-expm1f(2.0f * s.log_a)) * dg_sigmoid(gi) * u;
  return s;
}

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
  for (int t = t0; t < t1; ++t) {
    const DgStep s = dg_step(to_float<UT>(u[(long)t * ldu + c]), to_float<GT>(g[(long)t * ldg + gc]) + rb,
                             to_float<GT>(g[(long)t * ldg + gc + block]) + ib, dc);
    S = fmaf(s.a, S, s.x);
    const float v = y ? S * gelu_tanh(to_float<YT>(y[(long)t * ldy + y_off + c])) : S;
    out[(long)t * ldo + c] = from_float<OT>(v);
  }
  *st = S;
}

// Prompt portions: chunks of DG_C tokens counted from the portion's start, side by side.  The chunks of request r have the
// numbers cu_q[r] / DG_C + r and following.  A first pass leaves per chunk and channel what the chunk does to a state,
// S -> exp(L) S + X (the first chunk, whose state is known, leaves that state and its own end); the second puts the
// chunks before together, in order, and goes through the tokens again with the state that comes out.
// scratch: [3][chunks][C]: L, X (a first chunk's: its end), a first chunk's state at its start.
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
  float S = 0.f, L = 0.f;
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
      S = fmaf(expf(before[0]), S, before[plane]);
    }
  }
#pragma unroll 8
  for (int t = t0; t < t1; ++t) {
    const DgStep s = dg_step(to_float<UT>(u[(long)t * ldu + c]), to_float<GT>(g[(long)t * ldg + gc]) + rb,
                             to_float<GT>(g[(long)t * ldg + gc + block]) + ib, dc);
    S = fmaf(s.a, S, s.x);
    if (!LAST) {
      L += s.log_a;
    } else {
      const float v = y ? S * gelu_tanh(to_float<YT>(y[(long)t * ldy + y_off + c])) : S;
      out[(long)t * ldo + c] = from_float<OT>(v);
    }
  }
  if (!LAST) {
    mine[0] = L;
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
