// Causal attention over the paged cache whose scores are mixed over the heads before the softmax ("talking heads"):
//
//   score[h][j] = scale * sum_g talk[h][g] (q_g . k_(kv(g), j)),   kv(g) = g / (heads / kv heads)
//
// With the heads of one kv head taken together the sum over heads moves into the query:
//
//   score[h][j] = scale * sum_c (sum_{g of c} talk[h][g] q_g) . k_(c, j)
//
// so head h has one query of (kv heads x head size) entries against the row of all kv heads' keys of a token, and no score
// of one head ever waits for another's.  Head h reads the values of its own kv head.  A sink is a logit per head that
// joins the softmax's denominator.  Cache layout: see rope.hip.
#include "common.h"
#include "fmsamd.h"

#define TALK_THREADS 256

// One block per (head, token), float32 arithmetic whatever the storage: the true 32-bit path, and every size that the
// matrix-core kernels do not take.
template <typename T>
__global__ void __launch_bounds__(TALK_THREADS)
    talking_attn_generic_kernel(const T* __restrict__ q, long q_stride, T* __restrict__ out, long out_stride,
                                const int* __restrict__ positions, const int* __restrict__ seq_of_token,
                                const int* __restrict__ block_table, int table_stride, const T* __restrict__ k_cache,
                                const T* __restrict__ v_cache, const float* __restrict__ talk, const float* __restrict__ sink,
                                int nheads, int kvheads, int dim, int vdim, float scale, int window) {
  extern __shared__ float qm[];  // the mixed query: kvheads * dim
  __shared__ float ps[TALK_THREADS];
  __shared__ float scratch[17];
  const int h = blockIdx.x, t = blockIdx.y;
  const int seq = seq_of_token[t];
  T* o = out + (size_t)t * out_stride + (size_t)h * vdim;
  if (seq < 0) {
    for (int d = threadIdx.x; d < vdim; d += blockDim.x) o[d] = from_f32<T>(0.f);
    return;
  }
  const int pos = positions[t];
  const int lo = (window > 0 && pos - window + 1 > 0) ? pos - window + 1 : 0;
  const int n_keys = pos - lo + 1;
  const int per = nheads / kvheads;
  const int kh = h / per;
  const int* bt = block_table + (size_t)seq * table_stride;
  const size_t page_elems = (size_t)kvheads * PAGE_TOKENS * dim;
  const size_t vpage_elems = (size_t)kvheads * PAGE_TOKENS * vdim;
  const T* qrow = q + (size_t)t * q_stride;
  for (int i = threadIdx.x; i < kvheads * dim; i += blockDim.x) {
    const int c = i / dim, d = i % dim;
    float s = 0.f;
    for (int g = c * per; g < (c + 1) * per; ++g) s = fmaf(talk[(size_t)h * nheads + g], to_f32(qrow[(size_t)g * dim + d]), s);
    qm[i] = s;
  }
  __syncthreads();

  float m_run = -1e30f, l_run = 0.f, acc = 0.f;  // acc: this thread's output element d = threadIdx.x
  if (sink != nullptr) m_run = sink[h], l_run = 1.f;
  for (int base = 0; base < n_keys; base += TALK_THREADS) {
    const int u = base + threadIdx.x;
    float s = -INFINITY;
    if (u < n_keys) {
      const int j = lo + u;
      const T* page = k_cache + readable_page(bt[j / PAGE_TOKENS]) * page_elems + (size_t)(j % PAGE_TOKENS) * dim;
      float dot = 0.f;
      for (int c = 0; c < kvheads; ++c) {
        const T* krow = page + (size_t)c * PAGE_TOKENS * dim;
        for (int d = 0; d < dim; ++d) dot = fmaf(qm[c * dim + d], to_f32(krow[d]), dot);
      }
      s = dot * scale;
    }
    const float m_new = fmaxf(m_run, block_max(s, scratch));
    const float p = u < n_keys ? expf(s - m_new) : 0.f;
    const float alpha = expf(m_run - m_new);
    ps[threadIdx.x] = p;
    const float psum = block_sum(p, scratch);  // has the barriers that publish ps
    l_run = l_run * alpha + psum;
    m_run = m_new;
    if ((int)threadIdx.x < vdim) {
      float a = acc * alpha;
      const int n = n_keys - base < TALK_THREADS ? n_keys - base : TALK_THREADS;
      for (int i = 0; i < n; ++i) {
        const int j = lo + base + i;
        const T* vrow = v_cache + readable_page(bt[j / PAGE_TOKENS]) * vpage_elems + ((size_t)kh * vdim + threadIdx.x) * PAGE_TOKENS;
        a = fmaf(ps[i], to_f32(vrow[j % PAGE_TOKENS]), a);
      }
      acc = a;
    }
    __syncthreads();  // ps is overwritten by the next run of keys
  }
  if ((int)threadIdx.x < vdim) o[threadIdx.x] = from_f32<T>(l_run > 0.f ? acc / l_run : 0.f);
}

static int talking_common(const char* name, int n_tokens, int nheads, int kvheads, int dim, int vdim, long q_stride, long out_stride,
                          const void* talk) {
  FMS_REQUIRE(n_tokens > 0 && nheads > 0 && kvheads > 0 && nheads % kvheads == 0, "%s: %d heads over %d kv heads", name, nheads, kvheads);
  FMS_REQUIRE(dim > 0 && dim <= 256 && vdim > 0 && vdim <= 256, "%s: head sizes %d and %d (at most 256)", name, dim, vdim);
  FMS_REQUIRE(q_stride >= (long)nheads * dim && out_stride >= (long)nheads * vdim, "%s: rows too short", name);
  FMS_REQUIRE(talk != nullptr, "%s: the heads' mixing matrix is missing", name);
  return 0;
}

extern "C" int fmsamd_talking_attn_generic(const void* q, long q_stride, void* out, long out_stride, int dtype, const int* positions,
                                           const int* seq_of_token, const int* block_table, int table_stride, const void* k_cache,
                                           const void* v_cache, const float* talk, const float* sink, int n_tokens, int nheads,
                                           int kvheads, int head_dim, int value_dim, float scale, int window, hipStream_t stream) {
  if (n_tokens == 0) return 0;
  if (talking_common("talking_attn_generic", n_tokens, nheads, kvheads, head_dim, value_dim, q_stride, out_stride, talk)) return -1;
  FMS_REQUIRE(n_tokens <= 65535, "talking_attn_generic: %d tokens exceed one launch (65535)", n_tokens);
  const size_t lds = (size_t)kvheads * head_dim * sizeof(float);
  FMS_REQUIRE(lds <= 56 * 1024, "talking_attn_generic: %d kv heads of %d do not fit a block's LDS", kvheads, head_dim);
  const dim3 grid(nheads, n_tokens);
#define FMS_TG(T)                                                                                                                 \
  talking_attn_generic_kernel<T><<<grid, TALK_THREADS, lds, stream>>>((const T*)q, q_stride, (T*)out, out_stride, positions,      \
                                                                      seq_of_token, block_table, table_stride, (const T*)k_cache, \
                                                                      (const T*)v_cache, talk, sink, nheads, kvheads, head_dim,   \
                                                                      value_dim, scale, window)
  if (dtype == FMS_F32) FMS_TG(float);
  else if (dtype == FMS_BF16) FMS_TG(bf16);
  else FMS_REQUIRE(false, "talking_attn_generic: unknown dtype %d", dtype);
#undef FMS_TG
  FMS_LAUNCH_CHECK("talking_attn_generic");
  return 0;
}
