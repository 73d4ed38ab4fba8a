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
//   chunk_prep, chunk_scan, chunk_out: long steps, in chunks of 64 tokens as matrix products (float32 matrix instructions: true
//                32-bit products and sums).  With A(s, t) = prod of the decays of the tokens s + 1 .. t, channel by channel,
//                    o_t = S (A(start, t) q_t) + sum_{s <= t} M_ts v_s,    M_ts = sum_d q_td A(s, t)_d k_sd
//                    S  <- S diag(A(start, end)) + sum_s v_s (A(s, end) k_s)^T
//                chunk_prep makes every chunk's decayed queries, its M and what it adds to the state (chunks side by side,
//                nothing depends on the state).  A pair of tokens of two blocks of 16 decays as (from the later block's start to
//                t) (the blocks in between) (from s to its block's end), running products all of them, however small a decay is.
//                Pairs inside a block are quotients of such products, unless a channel's decay over the block is so small that
//                a quotient would leave the range: then they walk token by token.  One decay per head needs none of that:
//                M_ts = a^(t - s) q_t . k_s.
//                chunk_scan takes the states from chunk to chunk, element by element; chunk_out forms the outputs, chunks side
//                by side again, with norm and gate.
//
// The state is kept [slot][head][value channel][key channel], so that a lane's entries are contiguous.
#include "common.h"
#include "fmsamd.h"

#define LR_MAX_DIM 256

typedef fmsamd_linear_recurrence LinRec;

__device__ __forceinline__ f32x4 lr_zero4() { return f32x4{0.f, 0.f, 0.f, 0.f}; }

// sigmoid(z)^(inv_tau) = exp(-softplus(-z) inv_tau), softplus(x) = max(x, 0) + log(1 + exp(-|x|)).  What counts is the
// absolute error of the logarithm (it becomes the decay's relative one), so the hardware's exponential and logarithm serve.
__device__ __forceinline__ float lr_decay(float z, float inv_tau) {
  return __expf(-inv_tau * (fmaxf(-z, 0.f) + __logf(1.f + __expf(-fabsf(z)))));
}

// the gate's activation; silu, which every model here has, with the fast exponential where the result is rounded to 16 bits
template <typename T>
__device__ __forceinline__ float lr_gate(float x, int act) {
  if (sizeof(T) == 2 && act == FMS_ACT_SILU) return x * __builtin_amdgcn_rcpf(1.f + __expf(-x));
  return fms_activate(x, act);
}

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
    for (int i = tid; i < 2 * DP; i += blockDim.x) {
      const int which = i / DP, d = i % DP;
      float r = 0.f;
      if (d < D) {
        const float* src = x + (which == 0 ? a.col_q : a.col_k) + h * D;
        r = src[d];
        if (d < a.rot_dim) {
          const size_t at = lr_angle(a, a.positions[t], d);
          r = lr_turn(r, src[d ^ 1], d, a.cos_t[at], a.sin_t[at]);
        }
        if (which == 0) r *= a.q_scale;
      }
      lds[i] = r;
    }
    // decays: four lanes share a channel's sum; the second half of the block begins, the first has the queries and keys
    for (int i = tid ^ (blockDim.x >> 1); i < 4 * DP; i += blockDim.x) {
      const int d = i >> 2, quarter = i & 3;
      float r = 0.f;
      if (a.up_t != nullptr) {
        float z = 0.f;
        if (d < D) {
          const float* low = x + a.col_low;
          const float* up = a.up_t + h * D + d;
#pragma unroll 4
          for (int n = quarter; n < a.rank; n += 4) z = fmaf(up[(size_t)n * H * D], low[n], z);
        }
        z += __shfl_xor(z, 1, WAVE);
        z += __shfl_xor(z, 2, WAVE);
        if (d < D) r = lr_decay(z + a.up_bias[h * D + d], a.inv_tau);
      } else if (d < D) {
        r = expf(a.log_decay[h]);
      }
      if (quarter == 0) lds[2 * DP + d] = r;
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
        put(t, p, ys[p] * inv * (a.norm_w ? a.norm_w[p] : 1.f) * (a.out_dtype == FMS_F32 ? lr_gate<float>(g, a.act) : lr_gate<bf16>(g, a.act)));
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
#define LR_VALUES 128     // value channels at a time
#define LR_VALUE_LD 132   // and their LDS row
static_assert(LR_CHUNK * LR_VALUE_LD <= 2 * LR_CHUNK * LR_LD, "the values of a run take the place of queries and decays");
#define LR_RANK 32   // numbers of the low-rank projection at a time
#define LR_MAX_VDIM 256
// Every fourth turn of an unrolled loop over a lane's sixteen tokens: the compiler does not mix its turns beyond that (mixing all
// of them keeps every turn's temporaries in registers at once, and there are not enough of them for two waves).
#define LR_FOUR(i)                                            \
  do {                                                        \
    if (((i) & 3) == 3) __builtin_amdgcn_sched_barrier(0);    \
  } while (0)
#define LR_QUOTIENT_FROM 1e-24f  // a block's decay from which on pairs inside it may be formed as quotients

// What the kernels leave for one another, by chunk slot and head: M [64][64]; decayed queries [64][DP]; what the chunk adds to
// the state, S [V][DP], which the scan replaces by the state before the chunk; and the chunk's decay [DP].  DP: D rounded up to
// 16, zeros (decays: ones) from D on.  Chunk i of sequence b has the slot seq_starts[b] / 64 + b + i.
struct LrChunks {
  float *m, *q, *s, *end;
  int DP;
};
__device__ __forceinline__ size_t lr_chunk_slot(int start, int b, int i) { return (size_t)(start / LR_CHUNK + b + i); }

// The float32 product: lane (r = lane % 16, g = lane / 16) holds A[row r][k g] and B[k g][column r], and rows 4 g + i of
// column r of the result.  Which k a step takes is free as long as both operands agree: four steps take the k's
// 4 g + i, i = 0 .. 3, of sixteen, so that a lane's operands of four steps are four neighbours in memory.
#define LR_MFMA(a, b, c) __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0)

// SLICES: slices of 64 channels (D <= 64 SLICES)
template <bool PER_CHANNEL, int SLICES>
__global__ void __launch_bounds__(256, 2) lr_chunk_prep_kernel(LinRec a, LrChunks out) {
  // keys by slice; with a decay per channel to their block's end; then, of every slice, to the chunk's end
  __shared__ __attribute__((aligned(16))) float all_ks[SLICES][LR_CHUNK][LR_LD];
  __shared__ __attribute__((aligned(16))) float work[2][LR_CHUNK][LR_LD];
  float(*const qs)[LR_LD] = work[0];  // queries; with a decay per channel from their block's start
  float(*const as)[LR_LD] = work[1];  // a wave's own rows: the low-rank numbers, then keys over their block's decay up to them, or the decays themselves
  __shared__ __attribute__((aligned(16))) float tot[4][LR_SLICE];  // a block's decay
  // neighbouring blocks take neighbouring heads of the same tokens: together they read whole rows of memory
  const int h = blockIdx.x, chunk = blockIdx.y, b = blockIdx.z;
  const int start = a.seq_starts[b], t1 = a.seq_starts[b + 1];
  const int tc = start + chunk * LR_CHUNK;
  if (tc >= t1 || a.seq_of_token[start] < 0) return;
  const int n_tok = min(LR_CHUNK, t1 - tc);
  const int H = a.heads, D = a.dim, V = a.vdim, DP = out.DP;
  // the chunk's rows, and offsets inside them of 32 bits: a pointer for every row would take the registers of two waves
  const float* const rows = a.proj + (size_t)tc * a.ld;
  const unsigned ldp = (unsigned)a.ld;
  const int* const pos = a.positions + tc;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, r = lane & 15, g = lane >> 4;
  const size_t slot = lr_chunk_slot(start, b, chunk) * H + h;
  const float ld = PER_CHANNEL ? 0.f : a.log_decay[h];
  const int w0 = 16 * wave;  // the wave's tokens: w0 .. w0 + 15 of the chunk

  if constexpr (!PER_CHANNEL) {  // a token's decays to the chunk's ends, where decays per channel would be
    if (threadIdx.x < LR_CHUNK) {
      tot[0][threadIdx.x] = expf(ld * (float)(threadIdx.x + 1));
      tot[1][threadIdx.x] = expf(ld * (float)max(n_tok - 1 - (int)threadIdx.x, 0));
    }
    __syncthreads();
  }
  f32x4 mt[4];  // tile (wave, wave - jj) of M
#pragma unroll
  for (int j = 0; j < 4; ++j) mt[j] = lr_zero4();

#pragma unroll 1
  for (int slice = 0; slice * LR_SLICE < DP; ++slice) {
    const int d0 = slice * LR_SLICE, d = d0 + lane;
    const bool live = d < D;
    float(*const ks)[LR_LD] = all_ks[slice];
    float q[16], k[16], al[PER_CHANNEL ? 16 : 1];
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      const bool in = live && w0 + i < n_tok;
      const unsigned at = (unsigned)min(w0 + i, n_tok - 1) * ldp + (unsigned)(h * D + (live ? d : 0));
      const float qv = rows[at + a.col_q], kv = rows[at + a.col_k];
      q[i] = in ? qv : 0.f;  // past the sequence's end: a token that changes nothing
      k[i] = in ? kv : 0.f;
    }
    if constexpr (PER_CHANNEL) {
      float z[16];
      const float bias = live ? a.up_bias[h * D + d] : 0.f;
#pragma unroll
      for (int i = 0; i < 16; ++i) z[i] = bias;
      for (int n0 = 0; n0 < a.rank; n0 += LR_RANK) {
        const int nn = min(LR_RANK, a.rank - n0);
        const float* up = a.up_t + (size_t)n0 * H * D + h * D + (live ? d : 0);
        float u[16], lows[16 * LR_RANK / WAVE];
#pragma unroll
        for (int e = 0; e < 16; ++e) u[e] = up[(unsigned)(min(e, nn - 1) * H * D)];  // a number past the last meets a zero
#pragma unroll
        for (int e = 0; e < 16 * LR_RANK / WAVE; ++e) {
          const int tt = w0 + (e * WAVE + lane) / LR_RANK, n = lane % LR_RANK;
          const float v = rows[(unsigned)min(tt, n_tok - 1) * ldp + (unsigned)(a.col_low + n0 + min(n, nn - 1))];
          lows[e] = (n < nn && tt < n_tok) ? v : 0.f;
        }
        __builtin_amdgcn_wave_barrier();
#pragma unroll
        for (int e = 0; e < 16 * LR_RANK / WAVE; ++e) as[w0 + (e * WAVE + lane) / LR_RANK][lane % LR_RANK] = lows[e];
        __builtin_amdgcn_wave_barrier();
        for (int n = 0; n < nn; n += 16) {
          if (n > 0) {
#pragma unroll
            for (int e = 0; e < 16; ++e) u[e] = up[(unsigned)(min(n + e, nn - 1) * H * D)];
          }
#pragma unroll
          for (int i = 0; i < 16; ++i) {
#pragma unroll
            for (int c = 0; c < 4; ++c) {
              const f32x4 low = *reinterpret_cast<const f32x4*>(&as[w0 + i][n + 4 * c]);
#pragma unroll
              for (int e = 0; e < 4; ++e) z[i] = fmaf(u[4 * c + e], low[e], z[i]);
            }
            LR_FOUR(i);
          }
        }
      }
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        al[i] = (live && w0 + i < n_tok) ? lr_decay(z[i], a.inv_tau) : 1.f;
        LR_FOUR(i);
      }
    }
    if (d0 < a.rot_dim) {
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        const float qp = __shfl_xor(q[i], 1, WAVE), kp = __shfl_xor(k[i], 1, WAVE);
        if (d < a.rot_dim) {
          const unsigned at = (unsigned)lr_angle(a, pos[min(w0 + i, n_tok - 1)], d);
          const float c = a.cos_t[at], s = a.sin_t[at];
          q[i] = lr_turn(q[i], qp, d, c, s);
          k[i] = lr_turn(k[i], kp, d, c, s);
        }
        LR_FOUR(i);
      }
    }
#pragma unroll
    for (int i = 0; i < 16; ++i) q[i] *= a.q_scale;
    if (slice > 0) __syncthreads();  // the slice before is still being read
    bool quotients = true;
    if constexpr (PER_CHANNEL) {
      float run = 1.f;
#pragma unroll
      for (int i = 0; i < 16; ++i) run *= al[i];
      quotients = __all(run >= LR_QUOTIENT_FROM);
      if (!quotients) {
        // Pairs inside the block token by token: the lane of (key s = r, a quarter of the slice's channels) carries the key
        // along.  For decays that vanish within sixteen tokens only, where a quotient would leave the range.
#pragma unroll
        for (int i = 0; i < 16; ++i) {
          qs[w0 + i][lane] = q[i];
          ks[w0 + i][lane] = k[i];
          as[w0 + i][lane] = al[i];
        }
        __builtin_amdgcn_wave_barrier();
        f32x4 w[4];
#pragma unroll
        for (int c = 0; c < 4; ++c) w[c] = *reinterpret_cast<const f32x4*>(&ks[w0 + r][16 * g + 4 * c]);
#pragma unroll 1
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
          acc += __shfl_xor(acc, 16, WAVE);
          acc += __shfl_xor(acc, 32, WAVE);
#pragma unroll
          for (int i = 0; i < 4; ++i) mt[0][i] += t == 4 * g + i ? acc : 0.f;
        }
        __builtin_amdgcn_wave_barrier();
      }
      run = 1.f;
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        run *= al[i];
        q[i] *= run;
        qs[w0 + i][lane] = q[i];
        as[w0 + i][lane] = quotients ? k[i] * __builtin_amdgcn_rcpf(run) : 0.f;
        LR_FOUR(i);
      }
      tot[wave][lane] = run;
      run = 1.f;
#pragma unroll
      for (int i = 15; i >= 0; --i) {
        k[i] *= run;
        run *= al[i];
        ks[w0 + i][lane] = k[i];
      }
    } else {
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        qs[w0 + i][lane] = q[i];
        ks[w0 + i][lane] = k[i];
      }
    }
    __syncthreads();
    // products of the slice with the wave's own block and with the blocks before it
#pragma unroll
    for (int n = 0; n < LR_SLICE / 16; ++n) {
      f32x4 qv = *reinterpret_cast<const f32x4*>(&qs[w0 + r][16 * n + 4 * g]);
#pragma unroll
      for (int jj = 0; jj < 4; ++jj) {
        const int j = wave - jj;
        if (j >= 0) {  // uniform over the wave
          const float* krow = PER_CHANNEL && jj == 0 ? &as[w0 + r][16 * n + 4 * g] : &ks[16 * j + r][16 * n + 4 * g];
          const f32x4 kv = *reinterpret_cast<const f32x4*>(krow);
#pragma unroll
          for (int i = 0; i < 4; ++i) mt[jj] = LR_MFMA(qv[i], kv[i], mt[jj]);
          if (PER_CHANNEL && jj > 0) qv *= *reinterpret_cast<const f32x4*>(&tot[j][16 * n + 4 * g]);
        }
      }
    }
    // the decays to the chunk's ends: queries for the outputs, keys for the state
    float* const qo = out.q + slot * LR_CHUNK * DP;
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
        q[i] *= before;
        k[i] *= behind;
      }
      if (wave == 0 && d < DP) out.end[slot * DP + d] = all;
    } else {
#pragma unroll
      for (int i = 0; i < 16; ++i) {
        q[i] *= tot[0][w0 + i];
        k[i] *= tot[1][w0 + i];
      }
      if (wave == 0 && d < DP) out.end[slot * DP + d] = expf(ld * (float)n_tok);
    }
    if (d < DP) {
#pragma unroll
      for (int i = 0; i < 16; ++i) qo[(unsigned)((w0 + i) * DP + d)] = q[i];
    }
    __syncthreads();  // every wave has read the keys
#pragma unroll
    for (int i = 0; i < 16; ++i) ks[w0 + i][lane] = k[i];
  }
  float* const m = out.m + slot * (LR_CHUNK * LR_CHUNK);
#pragma unroll
  for (int jj = 0; jj < 4; ++jj) {
    const int j = wave - jj;
    if (j < 0) continue;
    const int s = 16 * j + r;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int t = w0 + 4 * g + i;
      float v = mt[jj][i];
      if constexpr (!PER_CHANNEL) v *= expf(ld * (float)max(t - s, 0));
      m[t * LR_CHUNK + s] = s <= t ? v : 0.f;
    }
  }
  // what the chunk adds to the state: values in runs of 128 channels through LDS; a wave has every fourth tile of 16 key channels
  float(*const vs)[LR_VALUE_LD] = reinterpret_cast<float(*)[LR_VALUE_LD]>(&work[0][0][0]);
  for (int v0 = 0; v0 < V; v0 += LR_VALUES) {
    float v[LR_CHUNK * LR_VALUES / 256];
#pragma unroll
    for (int e = 0; e < LR_CHUNK * LR_VALUES / 256; ++e) {
      const int tt = (e * 256 + (int)threadIdx.x) / LR_VALUES, p = v0 + (int)threadIdx.x % LR_VALUES;
      v[e] = rows[(unsigned)min(tt, n_tok - 1) * ldp + (unsigned)(a.col_v + h * V + min(p, V - 1))];  // past the end: meets zeros of the keys
    }
    __syncthreads();  // the queries, or the run before, are still being read
#pragma unroll
    for (int e = 0; e < LR_CHUNK * LR_VALUES / 256; ++e) vs[(e * 256 + threadIdx.x) / LR_VALUES][threadIdx.x % LR_VALUES] = v[e];
    __syncthreads();
    const int tiles = min(LR_VALUES / 16, (V - v0 + 15) / 16);
    for (int dt = wave; 16 * dt < DP; dt += 4) {
      float kk[4][4];
#pragma unroll
      for (int j = 0; j < 4; ++j) {
#pragma unroll
        for (int i = 0; i < 4; ++i) kk[j][i] = all_ks[dt / 4][16 * j + 4 * g + i][16 * (dt % 4) + r];
      }
      for (int pt = 0; pt < tiles; pt += 2) {
        f32x4 s0 = lr_zero4(), s1 = lr_zero4();
#pragma unroll
        for (int j = 0; j < 4; ++j) {
#pragma unroll
          for (int i = 0; i < 4; ++i) {
            s0 = LR_MFMA(kk[j][i], vs[16 * j + 4 * g + i][16 * pt + r], s0);
            s1 = LR_MFMA(kk[j][i], vs[16 * j + 4 * g + i][16 * pt + 16 + r], s1);
          }
        }
        const int pa = v0 + 16 * pt + r;
        float* dst = out.s + (slot * V + pa) * DP + 16 * dt + 4 * g;
        if (pa < V) *reinterpret_cast<f32x4*>(dst) = s0;
        if (pa + 16 < V) *reinterpret_cast<f32x4*>(dst + 16 * DP) = s1;
      }
    }
  }
}

// The states before every chunk, in the place of what the chunks add; a thread owns four key channels of a value channel.
#define LR_AHEAD 4  // chunks whose increments are asked for at a time
template <bool VEC>
__global__ void __launch_bounds__(256) lr_chunk_scan_kernel(LinRec a, LrChunks c) {
  const int b = blockIdx.z, h = blockIdx.y;
  const int t0 = a.seq_starts[b], t1 = a.seq_starts[b + 1];
  if (t0 >= t1 || a.seq_of_token[t0] < 0) return;
  const int D = a.dim, V = a.vdim, DP = c.DP, H = a.heads;
  const int item = blockIdx.x * 256 + threadIdx.x, per_row = DP / 4;
  const int p = item / per_row, d = (item % per_row) * 4;
  if (p >= V) return;
  float* const st = a.state + (((size_t)a.slot_ids[b] * H + h) * V + p) * D + d;
  f32x4 S;
  if (VEC) {
    S = d < D ? *reinterpret_cast<const f32x4*>(st) : lr_zero4();
  } else {
#pragma unroll
    for (int e = 0; e < 4; ++e) S[e] = d + e < D ? st[e] : 0.f;
  }
  const int chunks = (t1 - t0 + LR_CHUNK - 1) / LR_CHUNK;
  const size_t first = lr_chunk_slot(t0, b, 0);
  float* const s = c.s + ((first * H + h) * V + p) * DP + d;
  const float* const end = c.end + (first * H + h) * DP + d;
  const size_t step_s = (size_t)H * V * DP, step_e = (size_t)H * DP;
  for (int i0 = 0; i0 < chunks; i0 += LR_AHEAD) {
    f32x4 add[LR_AHEAD], e[LR_AHEAD];
#pragma unroll
    for (int i = 0; i < LR_AHEAD; ++i) {
      const int n = min(i0 + i, chunks - 1);
      add[i] = *reinterpret_cast<const f32x4*>(s + n * step_s);
      e[i] = *reinterpret_cast<const f32x4*>(end + n * step_e);
    }
#pragma unroll
    for (int i = 0; i < LR_AHEAD; ++i) {
      if (i0 + i < chunks) {
        *reinterpret_cast<f32x4*>(s + (i0 + i) * step_s) = S;
#pragma unroll
        for (int x = 0; x < 4; ++x) S[x] = fmaf(e[i][x], S[x], add[i][x]);
      }
    }
  }
  if (VEC) {
    if (d < D) *reinterpret_cast<f32x4*>(st) = S;
  } else {
#pragma unroll
    for (int e = 0; e < 4; ++e)
      if (d + e < D) st[e] = S[e];
  }
}

// The outputs of a chunk and head from the state before it, its decayed queries and its M; norm and gate included.  A wave has
// 16 tokens and all value channels (PT tiles of 16); the state goes through LDS, a slice of key channels at a time, the next
// one's on its way while this one is worked on.
template <int PT, typename T>
__global__ void __launch_bounds__(256, 2) lr_chunk_out_kernel(LinRec a, LrChunks c) {
  __shared__ __attribute__((aligned(16))) float ss[16 * PT][LR_LD];
  // neighbouring blocks take neighbouring heads of the same tokens: together they read whole rows of memory
  const int h = blockIdx.x, chunk = blockIdx.y, b = blockIdx.z;
  const int start = a.seq_starts[b], t1 = a.seq_starts[b + 1];
  const int tc = start + chunk * LR_CHUNK;
  if (tc >= t1 || a.seq_of_token[start] < 0) return;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, r = lane & 15, g = lane >> 4;
  const int w0 = 16 * wave;
  const int H = a.heads, V = a.vdim, DP = c.DP, n_tok = min(LR_CHUNK, t1 - tc);
  const size_t slot = lr_chunk_slot(start, b, chunk) * H + h;
  const float* const q = c.q + (slot * LR_CHUNK + w0 + r) * DP + 4 * g;
  const float* const s = c.s + slot * V * DP;
  const float* const m = c.m + slot * (LR_CHUNK * LR_CHUNK) + (w0 + r) * LR_CHUNK + 4 * g;
  const float* const rows = a.proj + (size_t)tc * a.ld;
  f32x4 y[PT];
#pragma unroll
  for (int p = 0; p < PT; ++p) y[p] = lr_zero4();

  // a thread moves four channels (4 (tid % 16) of the slice) of the rows tid / 16 + 16 i
  const int mrow = threadIdx.x >> 4, mcol = 4 * (threadIdx.x & 15);
  f32x4 next_s[PT], next_q[4];
  auto fetch = [&](int d0) {
#pragma unroll
    for (int i = 0; i < PT; ++i)  // a row past the last is the last: its sums are not used
      next_s[i] = d0 + mcol < DP ? *reinterpret_cast<const f32x4*>(s + (unsigned)(min(mrow + 16 * i, V - 1) * DP + d0 + mcol)) : lr_zero4();
#pragma unroll
    for (int n = 0; n < 4; ++n) next_q[n] = d0 + 16 * n < DP ? *reinterpret_cast<const f32x4*>(q + d0 + 16 * n) : lr_zero4();
  };
  struct Tokens {
    f32x4 m;
    float v[PT][4];
  };
  auto load_v = [&](Tokens& o, int j) {
    o.m = *reinterpret_cast<const f32x4*>(m + 16 * j);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const unsigned row = (unsigned)min(16 * j + 4 * g + i, n_tok - 1) * (unsigned)a.ld + (unsigned)(a.col_v + h * V);  // past the end: meets zeros of M
#pragma unroll
      for (int p = 0; p < PT; ++p) o.v[p][i] = rows[row + min(16 * p + r, V - 1)];
    }
  };
  auto work_v = [&](const Tokens& o) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
#pragma unroll
      for (int p = 0; p < PT; ++p) y[p] = LR_MFMA(o.m[i], o.v[p][i], y[p]);
    }
  };
  // Up to 128 value channels the tokens' first values are asked for ahead too (more of them leave no registers for that).
  constexpr bool AHEAD = PT <= 8;
  Tokens va, vb;
  fetch(0);
  if constexpr (AHEAD) load_v(va, 0);
  for (int d0 = 0; d0 < DP; d0 += LR_SLICE) {
    f32x4 qv[4];
#pragma unroll
    for (int n = 0; n < 4; ++n) qv[n] = next_q[n];
    if (d0 > 0) block_sync_lds();  // the slice before is still being read
#pragma unroll
    for (int i = 0; i < PT; ++i) *reinterpret_cast<f32x4*>(&ss[mrow + 16 * i][mcol]) = next_s[i];
    block_sync_lds();
    if (d0 + LR_SLICE < DP) fetch(d0 + LR_SLICE);
#pragma unroll
    for (int n = 0; n < 4; ++n) {
      constexpr int RUN = PT < 4 ? PT : 4;  // independent sums side by side
#pragma unroll
      for (int p0 = 0; p0 < PT; p0 += RUN) {
        f32x4 sv[RUN];
#pragma unroll
        for (int p = 0; p < RUN; ++p) sv[p] = *reinterpret_cast<const f32x4*>(&ss[16 * (p0 + p) + r][16 * n + 4 * g]);
#pragma unroll
        for (int i = 0; i < 4; ++i) {
#pragma unroll
          for (int p = 0; p < RUN; ++p) y[p0 + p] = LR_MFMA(qv[n][i], sv[p][i], y[p0 + p]);
        }
      }
    }
  }
  if constexpr (AHEAD) {
    for (int j = 0; j <= wave; j += 2) {  // tiles above the diagonal are not there
      load_v(vb, j + 1 <= wave ? j + 1 : j);
      work_v(va);
      if (j + 1 <= wave) {
        load_v(va, j + 2 <= wave ? j + 2 : j);
        work_v(vb);
      }
    }
  } else {
    for (int j = 0; j <= wave; ++j) {
      load_v(va, j);
      work_v(va);
    }
  }
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int t = tc + w0 + 4 * g + i;
    float sum = 0.f;
#pragma unroll
    for (int p = 0; p < PT; ++p)
      if (16 * p + r < V) sum = fmaf(y[p][i], y[p][i], sum);
    const float inv = a.out_scale / sqrtf(row16_sum(sum) / (float)V + a.eps);
    if (t < t1) {
      const float* gate = a.proj + (size_t)t * a.ld + a.col_g + (size_t)h * V;
      T* out = (T*)a.out + (size_t)t * a.ldo + (size_t)h * V;
#pragma unroll
      for (int p = 0; p < PT; ++p) {
        const int x = 16 * p + r;
        if (x < V) out[x] = from_f32<T>(y[p][i] * inv * (a.norm_w ? a.norm_w[x] : 1.f) * lr_gate<T>(gate[x], a.act));
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
  FMS_REQUIRE(a.out != nullptr && (a.out_dtype == FMS_F32 || a.out_dtype == FMS_BF16) && a.ldo >= hv, "%s: bad output", name);
  FMS_REQUIRE(a.act >= 0 && a.act <= FMS_ACT_LAST, "%s: unknown activation %d", name, a.act);
  FMS_REQUIRE(a.heads <= 65535 && a.n_seqs <= 65535, "%s: too many heads or sequences for one launch", name);
  return 0;
}

extern "C" int fmsamd_linear_recurrence_walk(const fmsamd_linear_recurrence* args, hipStream_t stream) {
  if (args->n_seqs == 0 || args->n_tokens == 0) return 0;
  const LinRec& a = *args;
  if (lr_check("linear_recurrence_walk", a)) return -1;
  const bool vec = a.dim % 4 == 0 && (uintptr_t)a.state % 16 == 0;
  const int K4 = a.dim <= 64 ? 1 : (a.dim <= 128 ? 2 : 4);
  const size_t lds = (size_t)(3 * 64 * K4 + a.vdim) * sizeof(float);
  FMS_REQUIRE(lds <= 64 * 1024, "linear_recurrence_walk: %d value channels do not fit the LDS", a.vdim);
  // Above 128 key channels a thread has registers for two rows of the state's (a head of more rows is then read in groups).
  const int threads = a.vdim <= 16 ? 256 : (a.vdim <= (K4 == 4 ? 32 : 128) ? 512 : 1024);
  const dim3 grid(a.heads, a.n_seqs);
#define FMS_LRW(K, TL)                                                            \
  do {                                                                            \
    if (vec) lr_walk_kernel<K, TL, true><<<grid, threads, lds, stream>>>(a);      \
    else lr_walk_kernel<K, TL, false><<<grid, threads, lds, stream>>>(a);         \
  } while (0)
#define FMS_LRT(K)                       \
  do {                                   \
    if (a.vdim <= 32) FMS_LRW(K, 1);     \
    else if (a.vdim <= 64) FMS_LRW(K, 2); \
    else FMS_LRW(K, 4);                  \
  } while (0)
  if (K4 == 1) FMS_LRT(1);
  else if (K4 == 2) FMS_LRT(2);
  else if (a.vdim <= 32) FMS_LRW(4, 1);
  else FMS_LRW(4, 2);
#undef FMS_LRT
#undef FMS_LRW
  FMS_LAUNCH_CHECK("linear_recurrence_walk");
  return 0;
}

static long lr_slots(int n_tokens, int n_seqs) { return n_tokens / LR_CHUNK + n_seqs + 1; }
static int lr_padded(int dim) { return (dim + 15) / 16 * 16; }

extern "C" long fmsamd_linear_recurrence_workspace(int n_tokens, int n_seqs, int heads, int dim, int vdim) {
  const long DP = lr_padded(dim);
  return lr_slots(n_tokens, n_seqs) * heads * (LR_CHUNK * LR_CHUNK + LR_CHUNK * DP + vdim * DP + DP) * (long)sizeof(float);
}

extern "C" int fmsamd_linear_recurrence_chunked(const fmsamd_linear_recurrence* args, int longest, float* workspace, long workspace_bytes,
                                                hipStream_t stream) {
  if (args->n_seqs == 0 || args->n_tokens == 0) return 0;
  const LinRec& a = *args;
  if (lr_check("linear_recurrence_chunked", a)) return -1;
  FMS_REQUIRE(a.ld * LR_CHUNK < (1L << 30) && (long)a.max_pos * a.rot_dim < (1L << 31), "linear_recurrence_chunked: rows or rotation tables too long");
  FMS_REQUIRE(a.vdim <= LR_MAX_VDIM, "linear_recurrence_chunked: %d value channels (at most %d)", a.vdim, LR_MAX_VDIM);
  FMS_REQUIRE(longest > 0 && longest <= a.n_tokens, "linear_recurrence_chunked: a longest sequence of %d in %d tokens", longest, a.n_tokens);
  FMS_REQUIRE(workspace != nullptr && (uintptr_t)workspace % 16 == 0 &&
                  workspace_bytes >= fmsamd_linear_recurrence_workspace(a.n_tokens, a.n_seqs, a.heads, a.dim, a.vdim),
              "linear_recurrence_chunked: the workspace is too small");
  const long rows = lr_slots(a.n_tokens, a.n_seqs) * a.heads;
  const int DP = lr_padded(a.dim);
  LrChunks c{};
  c.m = workspace;
  c.q = c.m + rows * LR_CHUNK * LR_CHUNK;
  c.s = c.q + rows * LR_CHUNK * DP;
  c.end = c.s + rows * a.vdim * DP;
  c.DP = DP;
  const dim3 grid(a.heads, ceil_div(longest, LR_CHUNK), a.n_seqs);
  FMS_REQUIRE(grid.y <= 65535, "linear_recurrence_chunked: a sequence of %d tokens exceeds one launch", longest);
#define FMS_LRP(SLICES)                                                                      \
  do {                                                                                       \
    if (a.up_t != nullptr) lr_chunk_prep_kernel<true, SLICES><<<grid, 256, 0, stream>>>(a, c); \
    else lr_chunk_prep_kernel<false, SLICES><<<grid, 256, 0, stream>>>(a, c);                \
  } while (0)
  if (DP <= 64) FMS_LRP(1);
  else if (DP <= 128) FMS_LRP(2);
  else FMS_LRP(4);
#undef FMS_LRP
  FMS_LAUNCH_CHECK("linear_recurrence chunk_prep");
  const dim3 scan(ceil_div((long)a.vdim * (DP / 4), 256), a.heads, a.n_seqs);
  if (a.dim % 4 == 0 && (uintptr_t)a.state % 16 == 0) lr_chunk_scan_kernel<true><<<scan, 256, 0, stream>>>(a, c);
  else lr_chunk_scan_kernel<false><<<scan, 256, 0, stream>>>(a, c);
  FMS_LAUNCH_CHECK("linear_recurrence chunk_scan");
#define FMS_LRO(PT)                                                                              \
  do {                                                                                           \
    if (a.out_dtype == FMS_F32) lr_chunk_out_kernel<PT, float><<<grid, 256, 0, stream>>>(a, c);  \
    else lr_chunk_out_kernel<PT, bf16><<<grid, 256, 0, stream>>>(a, c);                          \
  } while (0)
  if (a.vdim <= 16) FMS_LRO(1);
  else if (a.vdim <= 32) FMS_LRO(2);
  else if (a.vdim <= 64) FMS_LRO(4);
  else if (a.vdim <= 128) FMS_LRO(8);
  else FMS_LRO(16);
#undef FMS_LRO
  FMS_LAUNCH_CHECK("linear_recurrence chunk_out");
  return 0;
}
