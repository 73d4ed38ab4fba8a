// Linear attention with a decay: per head a matrix S [value channels V, key channels D],
//
//   S <- S diag(a) + v k^T,   o = S q            a: one number per head, or one per head and key channel
//
// with q and k of D channels, rotated by the token's position if the model says so (neighbouring pairs) and q scaled.  A
// decay per channel is sigmoid(z)^(1 / tau) with z = up (rank numbers of the token) + bias.  Every head's o is divided by its
// root mean square, times a weight (or none), times act(gate).  All in float32; only the result is rounded.
//
//   walk:        token by token, everything in one kernel: rotation, decays, recurrence, norm, gate (decode steps, short
//                portions).  A block owns a head of a sequence; 16 lanes share a row of S, four neighbouring entries a load.
//   chunk_prep, chunk_walk: long steps, in chunks of 64 tokens as matrix products (float32 matrix instructions: true 32-bit
//                products and sums).  With A(s, t) = prod of the decays of the tokens s + 1 .. t, channel by channel,
//                    o_t = S (A(start, t) q_t) + sum_{s <= t} M_ts v_s,    M_ts = sum_d q_td A(s, t)_d k_sd
//                    S  <- S diag(A(start, end)) + sum_s v_s (A(s, end) k_s)^T
//                chunk_prep makes every chunk's decayed queries and keys and its M (side by side, nothing depends on the
//                state).  Decays only ever multiply: inside blocks of 16 tokens as running products, and a pair of tokens of
//                two blocks as (from the later block's start to t) (blocks in between) (from s to its block's end), so that
//                no quotient and no large exponent appears however small a decay is.  Pairs inside a block of 16 walk: the
//                lane of (s, a quarter of the channels) carries k_s along, decayed from token to token.  One decay per head
//                needs none of that: M_ts = a^(t - s) q_t . k_s.
//                chunk_walk takes a sequence's chunks one after another with the state in accumulators, 16 value channels of
//                a head a block; norm and gate follow in a kernel of their own (gated_head_norm).
//
// The state is kept [slot][head][value channel][key channel], so that a lane's entries are contiguous.
#include "common.h"
#include "fmsamd.h"

#define LR_MAX_DIM 256

typedef fmsamd_linear_recurrence LinRec;

__device__ __forceinline__ f32x4 lr_zero4() { return f32x4{0.f, 0.f, 0.f, 0.f}; }

// sigmoid(z)^(inv_tau): the logarithm first, which keeps its digits where the sigmoid is close to one or to zero
__device__ __forceinline__ float lr_decay(float z, float inv_tau) { return expf(-softplus_f32(-z) * inv_tau); }

// Entry d of a row of a head, turned with its neighbour (x: the head's first entry).
__device__ __forceinline__ float lr_turn(float own, float other, int d, float c, float s) { return (d & 1) ? fmaf(s, other, c * own) : fmaf(c, own, -s * other); }

__device__ __forceinline__ size_t lr_angle(const LinRec& a, int pos, int d) {
  const int p = pos < 0 ? 0 : (pos < a.max_pos ? pos : a.max_pos - 1);  // the host has checked the range
  return (size_t)p * (a.rot_dim / 2) + d / 2;
}

// --------------------------------------------------------------------------
// token by token
// --------------------------------------------------------------------------
template <int K4, int TILES, bool VEC>
__global__ void __launch_bounds__(1024) lr_walk_kernel(LinRec a) {
  constexpr int DP = 64 * K4;
  extern __shared__ __attribute__((aligned(16))) float lds[];  // q | k | decays, DP entries each; then the head's outputs
  float* const ys = lds + 3 * DP;
  const int h = blockIdx.x, b = blockIdx.y, tid = threadIdx.x;
  const int H = a.heads, D = a.dim, V = a.vdim;
  const int t0 = uniform_load(a.seq_starts + b), t1 = uniform_load(a.seq_starts + b + 1);
  if (t0 >= t1) return;
  auto put = [&](int t, int p, float v) {
    const size_t at = (size_t)t * a.ldo + (size_t)h * V + p;
    if (a.out_dtype == FMS_F32) ((float*)a.out)[at] = v;
    else ((bf16*)a.out)[at] = from_f32<bf16>(v);
  };
  if (uniform_load(a.seq_of_token + t0) < 0) {  // a padding row of a step of fixed shape: zeros, which a product may read
    for (int t = t0; t < t1; ++t)
      for (int p = tid; p < V; p += blockDim.x) put(t, p, 0.f);
    return;
  }
  const int slot = uniform_load(a.slot_ids + b);
  const int part = tid & 15, row = tid >> 4, rows = blockDim.x >> 4;
  float* const st = a.state + ((size_t)slot * H + h) * V * D;
  const int groups = (V + rows * TILES - 1) / (rows * TILES);
  f32x4 S[TILES][K4];
  auto load = [&](int vg) {
#pragma unroll
    for (int i = 0; i < TILES; ++i) {
      const int p = (vg * TILES + i) * rows + row;
#pragma unroll
      for (int k = 0; k < K4; ++k) {
        const int d = 64 * k + 4 * part;
        const float* src = st + (size_t)p * D + d;
        if (VEC) {
          S[i][k] = (p < V && d < D) ? *reinterpret_cast<const f32x4*>(src) : lr_zero4();
        } else {
#pragma unroll
          for (int e = 0; e < 4; ++e) S[i][k][e] = (p < V && d + e < D) ? src[e] : 0.f;
        }
      }
    }
  };
  load(0);
  for (int t = t0; t < t1; ++t) {
    const float* x = a.proj + (size_t)t * a.ld;
    float v[TILES];
#pragma unroll
    for (int i = 0; i < TILES; ++i) v[i] = i * rows + row < V ? x[a.col_v + h * V + i * rows + row] : 0.f;
    const float gate = tid < V ? x[a.col_g + h * V + tid] : 0.f;
    for (int i = tid; i < 3 * DP; i += blockDim.x) {
      const int which = i / DP, d = i % DP;
      float r = 0.f;
      if (d < D) {
        if (which == 2) {
          if (a.up_t != nullptr) {
            float z = a.up_bias[h * D + d];
            const float* low = x + a.col_low;
            const float* up = a.up_t + h * D + d;
            for (int n = 0; n < a.rank; ++n) z = fmaf(up[(size_t)n * H * D], low[n], z);
            r = lr_decay(z, a.inv_tau);
          } else {
            r = expf(a.log_decay[h]);
          }
        } else {
          const float* src = x + (which == 0 ? a.col_q : a.col_k) + h * D;
          r = src[d];
          if (d < a.rot_dim) {
            const size_t at = lr_angle(a, a.positions[t], d);
            r = lr_turn(r, src[d ^ 1], d, a.cos_t[at], a.sin_t[at]);
          }
          if (which == 0) r *= a.q_scale;
        }
      }
      lds[i] = r;
    }
    __syncthreads();
    f32x4 q[K4], k[K4], al[K4];
#pragma unroll
    for (int n = 0; n < K4; ++n) {
      q[n] = *reinterpret_cast<const f32x4*>(lds + 64 * n + 4 * part);
      k[n] = *reinterpret_cast<const f32x4*>(lds + DP + 64 * n + 4 * part);
      al[n] = *reinterpret_cast<const f32x4*>(lds + 2 * DP + 64 * n + 4 * part);
    }
    for (int vg = 0; vg < groups; ++vg) {
      if (groups > 1 && (t > t0 || vg > 0)) load(vg);
#pragma unroll
      for (int i = 0; i < TILES; ++i) {
        const int p = (vg * TILES + i) * rows + row;
        const float vv = vg == 0 ? v[i] : (p < V ? x[a.col_v + h * V + p] : 0.f);
        float y = 0.f;
#pragma unroll
        for (int n = 0; n < K4; ++n) {
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            S[i][n][e] = fmaf(vv, k[n][e], al[n][e] * S[i][n][e]);
            y = fmaf(S[i][n][e], q[n][e], y);
          }
        }
        y = row16_sum(y);
        if (part == 0 && p < V) ys[p] = y;
        if ((groups > 1 || t == t1 - 1) && p < V) {
#pragma unroll
          for (int n = 0; n < K4; ++n) {
            const int d = 64 * n + 4 * part;
            float* dst = st + (size_t)p * D + d;
            if (VEC) {
              if (d < D) *reinterpret_cast<f32x4*>(dst) = S[i][n];
            } else {
#pragma unroll
              for (int e = 0; e < 4; ++e)
                if (d + e < D) dst[e] = S[i][n][e];
            }
          }
        }
      }
    }
    __syncthreads();
    if ((tid & ~63) < V) {  // whole waves
      float s = 0.f;
      for (int p = tid & 63; p < V; p += WAVE) s = fmaf(ys[p], ys[p], s);
      const float inv = a.out_scale / sqrtf(wave_sum(s) / (float)V + a.eps);
      for (int p = tid; p < V; p += blockDim.x) {
        const float g = p == tid ? gate : x[a.col_g + h * V + p];
        put(t, p, ys[p] * inv * (a.norm_w ? a.norm_w[p] : 1.f) * fms_activate(g, a.act));
      }
    }
    // the next token writes q, k and the decays, which every wave has read, and ys only behind the next barrier
  }
}

// --------------------------------------------------------------------------
// in chunks
// --------------------------------------------------------------------------
#define LR_CHUNK 64
#define LR_SLICE 64  // channels at a time: one a lane
#define LR_LD 68     // LDS row of a slice, padded
#define LR_RANK 32   // numbers of the low-rank projection at a time

// What chunk_prep leaves for the walk, by chunk slot and head: M [64][64], decayed queries and keys [64][DP] each, and the
// chunk's decay [DP]; DP: D rounded up to 16, zeros (decays: ones) from D on.  Chunk i of sequence b has the slot
// seq_starts[b] / 64 + b + i.
struct LrChunks {
  float *m, *q, *k, *end;
  int DP;
};
__device__ __forceinline__ size_t lr_chunk_slot(int start, int b, int i) { return (size_t)(start / LR_CHUNK + b + i); }

// The float32 product: lane (r = lane % 16, g = lane / 16) holds A[row r][k g] and B[k g][column r], and rows 4 g + i of
// column r of the result.  Which k a step takes is free as long as both operands agree: four steps take the k's
// 4 g + i, i = 0 .. 3, of sixteen, so that a lane's operands of four steps are four neighbours in memory.
#define LR_MFMA(a, b, c) __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0)

template <bool PER_CHANNEL>
__global__ void __launch_bounds__(256) lr_chunk_prep_kernel(LinRec a, LrChunks out) {
  __shared__ __attribute__((aligned(16))) float qs[LR_CHUNK][LR_LD];  // queries; with a decay per channel: as they are, then from their block's start
  __shared__ __attribute__((aligned(16))) float ks[LR_CHUNK][LR_LD];  // keys; ..., then to their block's end
  __shared__ __attribute__((aligned(16))) float as[PER_CHANNEL ? LR_CHUNK : 1][LR_LD];  // decays
  __shared__ __attribute__((aligned(16))) float tot[4][LR_SLICE];                       // a block's decay
  __shared__ float low[PER_CHANNEL ? LR_CHUNK : 1][LR_RANK];
  const int b = blockIdx.y, h = blockIdx.z;
  const int start = a.seq_starts[b], t1 = a.seq_starts[b + 1];
  const int tc = start + blockIdx.x * LR_CHUNK;
  if (tc >= t1 || a.seq_of_token[start] < 0) return;
  const int n_tok = min(LR_CHUNK, t1 - tc);
  const int H = a.heads, D = a.dim;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, r = lane & 15, g = lane >> 4;
  const size_t slot = lr_chunk_slot(start, b, blockIdx.x) * H + h;
  float* const qo = out.q + slot * LR_CHUNK * out.DP;
  float* const ko = out.k + slot * LR_CHUNK * out.DP;
  const float ld = PER_CHANNEL ? 0.f : a.log_decay[h];
  const int w0 = 16 * wave;  // the wave's tokens: w0 .. w0 + 15 of the chunk

  f32x4 mt[4];  // tile (wave, wave - jj) of M; with a decay per channel from jj = 1 on
#pragma unroll
  for (int j = 0; j < 4; ++j) mt[j] = lr_zero4();
  float diag[16];  // PER_CHANNEL: M[t][s = r], this lane's quarter of the channels
#pragma unroll
  for (int i = 0; i < 16; ++i) diag[i] = 0.f;

  for (int d0 = 0; d0 < out.DP; d0 += LR_SLICE) {
    const int d = d0 + lane;
    const bool live = d < D;
    float q[16], k[16], al[PER_CHANNEL ? 16 : 1];
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      const int t = tc + w0 + i;
      const bool in = live && t < t1;
      const float* x = a.proj + (size_t)(t < t1 ? t : tc) * a.ld + h * D + (live ? d : 0);
      q[i] = in ? x[a.col_q] : 0.f;  // past the sequence's end: a token that changes nothing
      k[i] = in ? x[a.col_k] : 0.f;
    }
    if (d0 < a.rot_dim) {
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        const int t = tc + w0 + i;
        const float qp = __shfl_xor(q[i], 1, WAVE), kp = __shfl_xor(k[i], 1, WAVE);
        if (d < a.rot_dim) {
          const size_t at = lr_angle(a, a.positions[t < t1 ? t : tc], d);
          const float c = a.cos_t[at], s = a.sin_t[at];
          q[i] = lr_turn(q[i], qp, d, c, s);
          k[i] = lr_turn(k[i], kp, d, c, s);
        }
      }
    }
#pragma unroll
    for (int i = 0; i < 16; ++i) q[i] *= a.q_scale;
    if constexpr (PER_CHANNEL) {
      float z[16];
      const float bias = live ? a.up_bias[h * D + d] : 0.f;
#pragma unroll
      for (int i = 0; i < 16; ++i) z[i] = bias;
      for (int n0 = 0; n0 < a.rank; n0 += LR_RANK) {
        const int nn = min(LR_RANK, a.rank - n0);
        __syncthreads();  // the slice before, or the numbers before, are still being read
        for (int i = threadIdx.x; i < LR_CHUNK * LR_RANK; i += 256) {
          const int tt = i / LR_RANK, n = i % LR_RANK;
          low[tt][n] = (n < nn && tt < n_tok) ? a.proj[(size_t)(tc + tt) * a.ld + a.col_low + n0 + n] : 0.f;
        }
        __syncthreads();
        const float* up = a.up_t + (size_t)n0 * H * D + h * D + (live ? d : 0);
        for (int n = 0; n < nn; ++n) {
          const float u = up[(size_t)n * H * D];
#pragma unroll
          for (int i = 0; i < 16; ++i) z[i] = fmaf(u, low[w0 + i][n], z[i]);
        }
      }
#pragma unroll
      for (int i = 0; i < 16; ++i) al[i] = (live && tc + w0 + i < t1) ? lr_decay(z[i], a.inv_tau) : 1.f;
    } else {
      __syncthreads();  // the slice before is still being read
    }
    // the wave's own rows of the slice: no other wave reads them before the barrier below
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      qs[w0 + i][lane] = q[i];
      ks[w0 + i][lane] = k[i];
      if constexpr (PER_CHANNEL) as[w0 + i][lane] = al[i];
    }
    if constexpr (PER_CHANNEL) {
      __builtin_amdgcn_wave_barrier();
      f32x4 w[4];
#pragma unroll
      for (int c = 0; c < 4; ++c) w[c] = *reinterpret_cast<const f32x4*>(&ks[w0 + r][16 * g + 4 * c]);
#pragma unroll
      for (int t = 0; t < 16; ++t) {
        float acc = 0.f;
#pragma unroll
        for (int c = 0; c < 4; ++c) {
          const f32x4 qv = *reinterpret_cast<const f32x4*>(&qs[w0 + t][16 * g + 4 * c]);
          const f32x4 av = *reinterpret_cast<const f32x4*>(&as[w0 + t][16 * g + 4 * c]);
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            w[c][e] = t > r ? w[c][e] * av[e] : w[c][e];
            acc = fmaf(qv[e], w[c][e], acc);
          }
        }
        diag[t] += acc;
      }
      __builtin_amdgcn_wave_barrier();
      float run = 1.f;
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        run *= al[i];
        q[i] *= run;
        qs[w0 + i][lane] = q[i];
      }
      tot[wave][lane] = run;
      run = 1.f;
#pragma unroll
      for (int i = 15; i >= 0; --i) {
        k[i] *= run;
        run *= al[i];
        ks[w0 + i][lane] = k[i];
      }
    }
    __syncthreads();
    // products of the slice with the blocks before the wave's own (and, with one decay per head, with its own)
#pragma unroll
    for (int n = 0; n < LR_SLICE / 16; ++n) {
      f32x4 qv = *reinterpret_cast<const f32x4*>(&qs[w0 + r][16 * n + 4 * g]);
#pragma unroll
      for (int jj = PER_CHANNEL ? 1 : 0; jj < 4; ++jj) {
        const int j = wave - jj;
        if (j >= 0) {  // uniform over the wave
          const f32x4 kv = *reinterpret_cast<const f32x4*>(&ks[16 * j + r][16 * n + 4 * g]);
#pragma unroll
          for (int i = 0; i < 4; ++i) mt[jj] = LR_MFMA(qv[i], kv[i], mt[jj]);
          if constexpr (PER_CHANNEL) qv *= *reinterpret_cast<const f32x4*>(&tot[j][16 * n + 4 * g]);
        }
      }
    }
    // decayed queries and keys for the walk
    if (d < out.DP) {
      if constexpr (PER_CHANNEL) {
        float before = 1.f, behind = 1.f, all = 1.f;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const float f = tot[j][lane];
          all *= f;
          if (j < wave) before *= f;
          if (j > wave) behind *= f;
        }
#pragma unroll
        for (int i = 0; i < 16; ++i) {
          qo[(size_t)(w0 + i) * out.DP + d] = q[i] * before;
          ko[(size_t)(w0 + i) * out.DP + d] = k[i] * behind;
        }
        if (wave == 0) out.end[slot * out.DP + d] = all;
      } else {
#pragma unroll
        for (int i = 0; i < 16; ++i) {
          const int s = w0 + i;
          qo[(size_t)s * out.DP + d] = q[i] * expf(ld * (float)(s + 1));
          ko[(size_t)s * out.DP + d] = k[i] * expf(ld * (float)max(n_tok - 1 - s, 0));
        }
        if (wave == 0) out.end[slot * out.DP + d] = expf(ld * (float)n_tok);
      }
    }
  }
  float* const m = out.m + slot * (LR_CHUNK * LR_CHUNK);
#pragma unroll
  for (int jj = 0; jj < 4; ++jj) {
    const int j = wave - jj;
    if (j < 0 || (PER_CHANNEL && jj == 0)) continue;
    const int s = 16 * j + r;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int t = w0 + 4 * g + i;
      float v = mt[jj][i];
      if constexpr (!PER_CHANNEL) v = s <= t ? v * expf(ld * (float)(t - s)) : 0.f;
      m[t * LR_CHUNK + s] = v;
    }
  }
  if constexpr (PER_CHANNEL) {
#pragma unroll
    for (int t = 0; t < 16; ++t) {
      float v = diag[t];
      v += __shfl_xor(v, 16, WAVE);
      v += __shfl_xor(v, 32, WAVE);
      if (g == t / 4) m[(w0 + t) * LR_CHUNK + w0 + r] = r <= t ? v : 0.f;
    }
  }
}

// KT: tiles of 16 key channels a wave owns (D <= 64 KT)
template <int KT, bool VEC>
__global__ void __launch_bounds__(256) lr_chunk_walk_kernel(LinRec a, LrChunks in, float* __restrict__ y, int p_tiles) {
  constexpr int NT = 4 * KT;
  __shared__ f32x4 states[2][NT * 64];  // the state as the chunk finds it: [tile][lane]
  // Blocks are dealt over the chip's eight dies in turn, each with a cache of its own: a head's blocks, which share its
  // queries, keys and M, go to one die.
  const int H = a.heads, per_seq = H * p_tiles;
  const int b = blockIdx.x / per_seq;
  int id = blockIdx.x % per_seq;
  if (H % 8 == 0) id = (id % 8) * (per_seq / 8) + id / 8;
  const int h = id / p_tiles, p0 = (id % p_tiles) * 16;
  const int t0 = a.seq_starts[b], t1 = a.seq_starts[b + 1];
  if (t0 >= t1 || a.seq_of_token[t0] < 0) return;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, r = lane & 15, g = lane >> 4;
  const int D = a.dim, V = a.vdim, DP = in.DP, last = t1 - 1;
  const int p = p0 + r;
  const bool live = p < V;
  const size_t col_v = (size_t)a.col_v + (size_t)h * V + (live ? p : 0);
  float* srow = a.state + (((size_t)a.slot_ids[b] * H + h) * V + (live ? p : 0)) * D;

  f32x4 S[KT];  // key channels 16 (wave + 4 k) + 4 g + i of value channel p
#pragma unroll
  for (int k = 0; k < KT; ++k) {
    const int d = 16 * (wave + 4 * k) + 4 * g;
    if (VEC) {
      S[k] = (live && d < D) ? *reinterpret_cast<const f32x4*>(srow + d) : lr_zero4();
    } else {
#pragma unroll
      for (int i = 0; i < 4; ++i) S[k][i] = (live && d + i < D) ? srow[d + i] : 0.f;
    }
  }

  struct Operands {
    f32x4 q[NT], m[4], end[KT];
    float v[4][4], k[KT][4][4];
  };
  auto load = [&](Operands& o, int chunk) {
    const int tc = t0 + chunk * LR_CHUNK;
    const size_t slot = lr_chunk_slot(t0, b, chunk) * H + h;
    const float* q = in.q + (slot * LR_CHUNK + 16 * wave + r) * DP + 4 * g;
#pragma unroll
    for (int n = 0; n < NT; ++n) o.q[n] = 16 * n < DP ? *reinterpret_cast<const f32x4*>(q + 16 * n) : lr_zero4();
    const float* m = in.m + slot * (LR_CHUNK * LR_CHUNK) + (16 * wave + r) * LR_CHUNK + 4 * g;
    const float* kk = in.k + slot * LR_CHUNK * DP;
    const float* end = in.end + slot * DP;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      o.m[j] = *reinterpret_cast<const f32x4*>(m + (j <= wave ? 16 * j : 0));  // tiles above the diagonal are not there
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        o.v[j][i] = a.proj[(size_t)min(tc + 16 * j + 4 * g + i, last) * a.ld + col_v];  // past the end: meets zeros of M and k
#pragma unroll
        for (int k = 0; k < KT; ++k) {
          const int d = 16 * (wave + 4 * k) + r;
          o.k[k][j][i] = d < DP ? kk[(size_t)(16 * j + 4 * g + i) * DP + d] : 0.f;
        }
      }
    }
#pragma unroll
    for (int k = 0; k < KT; ++k) {
      const int d = 16 * (wave + 4 * k) + 4 * g;
      o.end[k] = d < DP ? *reinterpret_cast<const f32x4*>(end + d) : lr_zero4();
    }
  };
  auto work = [&](const Operands& o, int chunk) {
    f32x4* st = states[chunk & 1];  // the other buffer may still be read by a wave of the chunk before
#pragma unroll
    for (int k = 0; k < KT; ++k) st[(wave + 4 * k) * 64 + lane] = S[k];
    block_sync_lds();
    f32x4 y0 = lr_zero4(), y1 = lr_zero4();
#pragma unroll
    for (int n = 0; n < NT; n += 2) {
      const f32x4 s0 = st[n * 64 + lane], s1 = st[(n + 1) * 64 + lane];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        y0 = LR_MFMA(o.q[n][i], s0[i], y0);
        y1 = LR_MFMA(o.q[n + 1][i], s1[i], y1);
      }
    }
    f32x4 out = y0 + y1;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      if (j <= wave) {  // uniform over the wave
#pragma unroll
        for (int i = 0; i < 4; ++i) out = LR_MFMA(o.m[j][i], o.v[j][i], out);
      }
    }
#pragma unroll
    for (int k = 0; k < KT; ++k) S[k] *= o.end[k];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
#pragma unroll
      for (int i = 0; i < 4; ++i) {
#pragma unroll
        for (int k = 0; k < KT; ++k) S[k] = LR_MFMA(o.k[k][j][i], o.v[j][i], S[k]);
      }
    }
    const int t = t0 + chunk * LR_CHUNK + 16 * wave + 4 * g;
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (live && t + i <= last) y[(size_t)(t + i) * H * V + (size_t)h * V + p] = out[i];
  };
  // the next chunk's operands are asked for before this one is worked on
  const int chunks = (t1 - t0 + LR_CHUNK - 1) / LR_CHUNK;
  Operands oa, ob;
  load(oa, 0);
  for (int c = 0; c < chunks; c += 2) {
    load(ob, c + 1 < chunks ? c + 1 : c);
    work(oa, c);
    if (c + 1 < chunks) {
      load(oa, c + 2 < chunks ? c + 2 : c + 1);
      work(ob, c + 1);
    }
  }
  if (live) {
#pragma unroll
    for (int k = 0; k < KT; ++k) {
      const int d = 16 * (wave + 4 * k) + 4 * g;
      if (VEC) {
        if (d < D) *reinterpret_cast<f32x4*>(srow + d) = S[k];
      } else {
#pragma unroll
        for (int i = 0; i < 4; ++i)
          if (d + i < D) srow[d + i] = S[k][i];
      }
    }
  }
}

// --------------------------------------------------------------------------
static int lr_check(const char* name, const LinRec& a) {
  FMS_REQUIRE(a.n_seqs > 0 && a.n_tokens > 0 && a.heads > 0 && a.dim > 0 && a.dim <= LR_MAX_DIM && a.vdim > 0,
              "%s: bad sizes seqs=%d tokens=%d heads=%d dim=%d (at most %d) vdim=%d", name, a.n_seqs, a.n_tokens, a.heads, a.dim, LR_MAX_DIM, a.vdim);
  const long hd = (long)a.heads * a.dim, hv = (long)a.heads * a.vdim;
  FMS_REQUIRE(a.col_q >= 0 && a.col_q + hd <= a.ld && a.col_k >= 0 && a.col_k + hd <= a.ld && a.col_v >= 0 && a.col_v + hv <= a.ld &&
                  a.col_g >= 0 && a.col_g + hv <= a.ld, "%s: the rows do not hold the columns asked for", name);
  FMS_REQUIRE((a.up_t != nullptr) != (a.log_decay != nullptr), "%s: decays are given either per head or by a projection", name);
  FMS_REQUIRE(a.up_t == nullptr || (a.rank > 0 && a.up_bias != nullptr && a.col_low >= 0 && a.col_low + a.rank <= a.ld),
              "%s: a decay through %d numbers", name, a.rank);
  FMS_REQUIRE(a.rot_dim >= 0 && a.rot_dim % 2 == 0 && a.rot_dim <= a.dim &&
                  (a.rot_dim == 0 || (a.cos_t != nullptr && a.sin_t != nullptr && a.positions != nullptr && a.max_pos > 0)),
              "%s: %d rotated channels of %d", name, a.rot_dim, a.dim);
  FMS_REQUIRE(a.heads <= 65535 && a.n_seqs <= 65535, "%s: too many heads or sequences for one launch", name);
  return 0;
}

extern "C" int fmsamd_linear_recurrence_walk(const fmsamd_linear_recurrence* args, hipStream_t stream) {
  if (args->n_seqs == 0 || args->n_tokens == 0) return 0;
  const LinRec& a = *args;
  if (lr_check("linear_recurrence_walk", a)) return -1;
  FMS_REQUIRE(a.out != nullptr && (a.out_dtype == FMS_F32 || a.out_dtype == FMS_BF16) && a.ldo >= (long)a.heads * a.vdim,
              "linear_recurrence_walk: bad output");
  FMS_REQUIRE(a.act >= 0 && a.act <= FMS_ACT_LAST, "linear_recurrence_walk: unknown activation %d", a.act);
  const bool vec = a.dim % 4 == 0 && (uintptr_t)a.state % 16 == 0;
  const int K4 = a.dim <= 64 ? 1 : (a.dim <= 128 ? 2 : 4);
  const size_t lds = (size_t)(3 * 64 * K4 + a.vdim) * sizeof(float);
  FMS_REQUIRE(lds <= 64 * 1024, "linear_recurrence_walk: %d value channels do not fit the LDS", a.vdim);
  const int threads = a.vdim <= 16 ? 256 : (a.vdim <= 32 ? 512 : 1024);
  const dim3 grid(a.heads, a.n_seqs);
#define FMS_LRW(K, TL)                                                            \
  do {                                                                            \
    if (vec) lr_walk_kernel<K, TL, true><<<grid, threads, lds, stream>>>(a);      \
    else lr_walk_kernel<K, TL, false><<<grid, threads, lds, stream>>>(a);         \
  } while (0)
#define FMS_LRT(K)                       \
  do {                                   \
    if (a.vdim <= 64) FMS_LRW(K, 1);     \
    else if (a.vdim <= 128) FMS_LRW(K, 2); \
    else FMS_LRW(K, 4);                  \
  } while (0)
  if (K4 == 1) FMS_LRT(1);
  else if (K4 == 2) FMS_LRT(2);
  else FMS_LRT(4);
#undef FMS_LRT
#undef FMS_LRW
  FMS_LAUNCH_CHECK("linear_recurrence_walk");
  return 0;
}

static long lr_slots(int n_tokens, int n_seqs) { return n_tokens / LR_CHUNK + n_seqs + 1; }
static int lr_padded(int dim) { return (dim + 15) / 16 * 16; }

extern "C" long fmsamd_linear_recurrence_workspace(int n_tokens, int n_seqs, int heads, int dim) {
  const long DP = lr_padded(dim);
  return lr_slots(n_tokens, n_seqs) * heads * (LR_CHUNK * LR_CHUNK + 2 * LR_CHUNK * DP + DP) * (long)sizeof(float);
}

// y float32 [n_tokens, heads * vdim]: the heads as the recurrence leaves them (no norm, no gate)
extern "C" int fmsamd_linear_recurrence_chunked(const fmsamd_linear_recurrence* args, float* y, int longest, float* workspace,
                                                long workspace_bytes, hipStream_t stream) {
  if (args->n_seqs == 0 || args->n_tokens == 0) return 0;
  const LinRec& a = *args;
  if (lr_check("linear_recurrence_chunked", a)) return -1;
  FMS_REQUIRE(longest > 0 && longest <= a.n_tokens, "linear_recurrence_chunked: a longest sequence of %d in %d tokens", longest, a.n_tokens);
  FMS_REQUIRE(y != nullptr && workspace != nullptr && (uintptr_t)workspace % 16 == 0 &&
                  workspace_bytes >= fmsamd_linear_recurrence_workspace(a.n_tokens, a.n_seqs, a.heads, a.dim),
              "linear_recurrence_chunked: the workspace is too small");
  const long rows = lr_slots(a.n_tokens, a.n_seqs) * a.heads;
  const int DP = lr_padded(a.dim);
  LrChunks c{};
  c.m = workspace;
  c.q = c.m + rows * LR_CHUNK * LR_CHUNK;
  c.k = c.q + rows * LR_CHUNK * DP;
  c.end = c.k + rows * LR_CHUNK * DP;
  c.DP = DP;
  const dim3 grid(ceil_div(longest, LR_CHUNK), a.n_seqs, a.heads);
  if (a.up_t != nullptr) lr_chunk_prep_kernel<true><<<grid, 256, 0, stream>>>(a, c);
  else lr_chunk_prep_kernel<false><<<grid, 256, 0, stream>>>(a, c);
  FMS_LAUNCH_CHECK("linear_recurrence chunk_prep");
  const int p_tiles = ceil_div(a.vdim, 16);
  const long blocks = (long)a.n_seqs * a.heads * p_tiles;
  FMS_REQUIRE(blocks < (1L << 31), "linear_recurrence_chunked: too many blocks");
  const bool vec = a.dim % 4 == 0 && (uintptr_t)a.state % 16 == 0;
#define FMS_LRC(KT)                                                                                          \
  do {                                                                                                       \
    if (vec) lr_chunk_walk_kernel<KT, true><<<(unsigned)blocks, 256, 0, stream>>>(a, c, y, p_tiles);         \
    else lr_chunk_walk_kernel<KT, false><<<(unsigned)blocks, 256, 0, stream>>>(a, c, y, p_tiles);            \
  } while (0)
  if (a.dim <= 64) FMS_LRC(1);
  else if (a.dim <= 128) FMS_LRC(2);
  else FMS_LRC(4);
#undef FMS_LRC
  FMS_LAUNCH_CHECK("linear_recurrence chunk_walk");
  return 0;
}
