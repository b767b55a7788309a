// Paged key/value store and the general paged causal attention kernel.
//
// A page pool of one cache slot holds keys (or values) as
//   [num_pages][n_kv_head][page_size][head_dim].
// New keys and values are stored after projection, unscaled, before attention
// reads them (reference: src/minigpt_infer/model.py:55-59,
// src/minigpt_infer/cache/paged.py:125-137).
//
// attention: S = q k^T * scale; a query at absolute position p sees the keys at
// positions max(0, p-window+1)..p of its own request (window 0 = all of them);
// softmax over keys in 32-bit (with `sinks`, one more term exp(sinks[head]) in its denominator that
// has no value; with `softcap` > 0 every score becomes softcap * tanh(score / softcap) first; with `gate`
// a head's output is multiplied by sigmoid(gate[token][head]));
// with `keep_first` > 0 a query behind a window also sees the keys at positions below keep_first; with
// `score_bias` (a number per head) there is no softmax: a visible key's weight is
// sigmoid(score + score_bias[head]), and the weights are not normalised;
// with `chunked` a query sees the positions of its own chunk of `window` positions instead of the last `window`;
// with `dist_bias` ([heads][bias_len]) the number for the key's distance is added to the scaled score;
// with `slopes` ([heads]) slope * distance is taken off the scaled (and capped) score;
// y = P v (reference: src/minigpt_infer/model.py:61-87,
// the rule col <= cache_len + row of src/minigpt_infer/batch.py:202-227).
//
// The general kernel runs one wave per (token, head).  Keys are reduced in
// chunks of 64 that start at absolute positions that are multiples of 64, so the
// order of the sums for a query depends only on its position, never on how the
// tokens were cut into steps or what else is in the batch.  Slots outside
// [begin, end) are never loaded.
#include "attention_mask.h"
#include "common.h"
#include "launchers.h"

template <typename T>
__global__ void kv_write_kernel(const T* __restrict__ qkv, long ld, int k_off, int v_off,
                                T* __restrict__ kpool, T* __restrict__ vpool,
                                const int* __restrict__ slot_mapping, int n_tokens, int n_kv_head,
                                int head_dim, int page_size) {
  int n = blockIdx.x;
  if (n >= n_tokens) return;
  int slot = slot_mapping[n];
  if (slot < 0) return;  // padded row
  long page = slot / page_size;
  int off = slot - (int)page * page_size;
  const T* src = qkv + (long)n * ld;
  int width = n_kv_head * head_dim;
  for (int c = threadIdx.x; c < width; c += blockDim.x) {
    int h = c / head_dim, d = c - h * head_dim;
    long dst = ((page * n_kv_head + h) * page_size + off) * (long)head_dim + d;
    kpool[dst] = src[k_off + c];
    vpool[dst] = src[v_off + c];
  }
}

extern "C" int mgpt_kv_write(const void* qkv, int dtype, long ld, int k_off, int v_off, void* kpool,
                             void* vpool, const int* slot_mapping, int n_tokens, int n_kv_head,
                             int head_dim, int page_size, hipStream_t stream) {
  if (n_tokens == 0) return MGPT_OK;
  if (!qkv || !kpool || !vpool || !slot_mapping) return MGPT_ERR_NULL;
  if (n_tokens < 0 || n_kv_head <= 0 || head_dim <= 0 || page_size <= 0) return MGPT_ERR_BAD_SHAPE;
  int width = n_kv_head * head_dim;
  int threads = width >= 256 ? 256 : 64;
  if (dtype == MGPT_F32) {
    hipLaunchKernelGGL(kv_write_kernel<float>, dim3(n_tokens), dim3(threads), 0, stream,
                       (const float*)qkv, ld, k_off, v_off, (float*)kpool, (float*)vpool,
                       slot_mapping, n_tokens, n_kv_head, head_dim, page_size);
  } else if (dtype == MGPT_BF16) {
    hipLaunchKernelGGL(kv_write_kernel<bf16_t>, dim3(n_tokens), dim3(threads), 0, stream,
                       (const bf16_t*)qkv, ld, k_off, v_off, (bf16_t*)kpool, (bf16_t*)vpool,
                       slot_mapping, n_tokens, n_kv_head, head_dim, page_size);
  } else {
    return MGPT_ERR_BAD_DTYPE;
  }
  return mgpt_last_error();
}

#define MAX_DPL 16  // head_dim <= 1024

template <typename T, bool FAST_EXP>
__global__ __launch_bounds__(64) void paged_attention_generic_kernel(
    const T* __restrict__ q, long ldq, T* __restrict__ out, long ldo, const T* __restrict__ kpool,
    const T* __restrict__ vpool, const int* __restrict__ block_tables, int max_blocks,
    const int* __restrict__ cu_q, const int* __restrict__ seq_lens, const int* __restrict__ q_req,
    int n_tokens, int n_head, int n_kv_head, int head_dim, int page_size, float scale, int window,
    const float* __restrict__ sinks, float softcap, const T* __restrict__ gate, long ldg, int keep_first,
    const float* __restrict__ score_bias, int chunked, const float* __restrict__ dist_bias, int bias_len,
    const float* __restrict__ slopes) {
  __shared__ float q_s[MAX_DPL * MGPT_WAVE];
  __shared__ float p_s[MGPT_WAVE];
  __shared__ int page_s[MGPT_WAVE];

  const int n = blockIdx.x, h = blockIdx.y, lane = threadIdx.x;
  if (n >= n_tokens) return;
  const int r = q_req[n];
  if (r < 0) return;  // padded token
  const int seq_len = seq_lens[r];
  const int q_start = cu_q[r], q_len = cu_q[r + 1] - q_start;
  const int qpos = seq_len - q_len + (n - q_start);
  const int kv_end = qpos + 1;
  const int kv_begin = first_seen(qpos, window, chunked);
  const int hk = h / (n_head / n_kv_head);
  const int* bt = block_tables + (long)r * max_blocks;

  for (int d = lane; d < head_dim; d += MGPT_WAVE)
    q_s[d] = to_float<T>(q[(long)n * ldq + (long)h * head_dim + d]);
  __syncthreads();

  float m = -INFINITY, l = 0.f;
  float acc[MAX_DPL];
#pragma unroll
  for (int i = 0; i < MAX_DPL; ++i) acc[i] = 0.f;

  const bool weigh = score_bias != nullptr;   // sigmoid weights, no softmax
  const float bias = weigh ? score_bias[h] : 0.f;
  for (int c0 = 0; c0 < kv_end; c0 += MGPT_WAVE) {
    if (c0 + MGPT_WAVE <= kv_begin && c0 >= keep_first) {   // behind the kept first keys, before the window: on to the window's chunk
      c0 = (kv_begin / MGPT_WAVE) * MGPT_WAVE - MGPT_WAVE;
      continue;
    }
    const int j = c0 + lane;
    const bool valid = (j >= kv_begin || j < keep_first) && (j < kv_end);
    float s = -INFINITY;
    int page = -1;
    if (valid) {
      page = bt[j / page_size];
      const int off = j % page_size;
      const T* kr = kpool + (((long)page * n_kv_head + hk) * page_size + off) * (long)head_dim;
      float dot = 0.f;
      for (int d = 0; d < head_dim; ++d) dot = fmaf(q_s[d], to_float<T>(kr[d]), dot);
      s = dot * scale;
      if (dist_bias) s += dist_bias[(long)h * bias_len + distance_entry(qpos - j, bias_len)];
      if (softcap > 0.f) s = softcap * tanhf(s / softcap);
      if (slopes) s -= slopes[h] * (float)(qpos - j);
    }
    float p = 0.f, alpha = 1.f;
    if (weigh) {
      if (valid) p = 1.0f / (1.0f + (FAST_EXP ? __expf(-(s + bias)) : expf(-(s + bias))));
    } else {
      const float m_new = fmaxf(m, wave_max(s));
      if (valid) p = FAST_EXP ? __expf(s - m_new) : expf(s - m_new);
      alpha = (m == -INFINITY) ? 0.f : (FAST_EXP ? __expf(m - m_new) : expf(m - m_new));
      l = l * alpha + wave_sum(p);
      m = m_new;
    }
    __syncthreads();  // previous chunk's readers of p_s / page_s are done
    p_s[lane] = p;
    page_s[lane] = page;
    __syncthreads();
    const int j_hi = (kv_end < c0 + MGPT_WAVE ? kv_end : c0 + MGPT_WAVE) - c0;
#pragma unroll
    for (int i = 0; i < MAX_DPL; ++i) {
      const int d = lane + i * MGPT_WAVE;
      if (d < head_dim) {
        float a = acc[i] * alpha;
        for (int jj = 0; jj < j_hi; ++jj) {
          if (page_s[jj] < 0) continue;   // a key that the query does not see
          const int off = (c0 + jj) % page_size;
          const T* vr = vpool + (((long)page_s[jj] * n_kv_head + hk) * page_size + off) * (long)head_dim;
          a = fmaf(p_s[jj], to_float<T>(vr[d]), a);
        }
        acc[i] = a;
      }
    }
  }
  if (sinks) {
    // one more term in the denominator, exp(sink), with no key and no value
    const float sink = sinks[h];
    const float m_new = fmaxf(m, sink);
    const float alpha = FAST_EXP ? __expf(m - m_new) : expf(m - m_new);
    l = l * alpha + (FAST_EXP ? __expf(sink - m_new) : expf(sink - m_new));
#pragma unroll
    for (int i = 0; i < MAX_DPL; ++i) acc[i] *= alpha;
  }
  float inv_l = weigh ? 1.0f : 1.0f / l;
  if (gate) {   // the head's output times sigmoid(gate[token][head])
    const float gv = to_float<T>(gate[(long)n * ldg + h]);
    inv_l *= 1.0f / (1.0f + (FAST_EXP ? __expf(-gv) : expf(-gv)));
  }
#pragma unroll
  for (int i = 0; i < MAX_DPL; ++i) {
    const int d = lane + i * MGPT_WAVE;
    if (d < head_dim) out[(long)n * ldo + (long)h * head_dim + d] = from_float<T>(acc[i] * inv_l);
  }
}

// q: [n_tokens, n_head*head_dim] with row stride ldq; out likewise with ldo.
// q_req[t] = index of token t's request in this step (or -1 for a padded token),
// cu_q[r]..cu_q[r+1] = the tokens of request r, seq_lens[r] = its length after this step.
extern "C" int mgpt_paged_attention_generic(
    const void* q, long ldq, void* out, long ldo, const void* kpool, const void* vpool,
    const int* block_tables, int max_blocks, const int* cu_q, const int* seq_lens, const int* q_req,
    int n_tokens, int n_head, int n_kv_head, int head_dim, int page_size, float scale, int window,
    int dtype, int fast_exp, const float* sinks, float softcap, const void* gate, long ldg, int keep_first,
    const float* score_bias, int chunked, const float* dist_bias, int bias_len, const float* slopes,
    hipStream_t stream) {
  if (n_tokens == 0) return MGPT_OK;
  if (!q || !out || !kpool || !vpool || !block_tables || !cu_q || !seq_lens || !q_req) return MGPT_ERR_NULL;
  if (n_tokens < 0 || n_head <= 0 || n_kv_head <= 0 || (n_head % n_kv_head) != 0 || head_dim <= 0 ||
      head_dim > MAX_DPL * MGPT_WAVE || page_size <= 0 || max_blocks <= 0 || window < 0 || keep_first < 0 || (score_bias && (sinks || softcap > 0.f)) ||
      (dist_bias && (bias_len <= 0 || score_bias || softcap > 0.f)) || (slopes && (dist_bias || score_bias)))
    return MGPT_ERR_BAD_SHAPE;
  if (n_head > 65535) return MGPT_ERR_TOO_LARGE;
  if (window == 0) keep_first = 0;   // every key is seen anyway
  dim3 grid(n_tokens, n_head), block(MGPT_WAVE);
#define LAUNCH(T, F)                                                                              \
  hipLaunchKernelGGL((paged_attention_generic_kernel<T, F>), grid, block, 0, stream, (const T*)q, ldq, \
                     (T*)out, ldo, (const T*)kpool, (const T*)vpool, block_tables, max_blocks, cu_q,  \
                     seq_lens, q_req, n_tokens, n_head, n_kv_head, head_dim, page_size, scale, window, sinks, softcap, \
                     (const T*)gate, ldg, keep_first, score_bias, chunked, dist_bias, bias_len, slopes)
  if (dtype == MGPT_F32) {
    if (fast_exp) LAUNCH(float, true); else LAUNCH(float, false);
  } else if (dtype == MGPT_BF16) {
    if (fast_exp) LAUNCH(bf16_t, true); else LAUNCH(bf16_t, false);
  } else {
    return MGPT_ERR_BAD_DTYPE;
  }
#undef LAUNCH
  return mgpt_last_error();
}
