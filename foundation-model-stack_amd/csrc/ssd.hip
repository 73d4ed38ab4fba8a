// The state-space recurrence of Mamba-2: per head a matrix S [value channels P, state rows N],
//
//   S <- exp(-exp(a_log) d) S + d x B^T,   y = S C + skip x,   d = softplus(dt + dt_bias)
//
// with x of P channels per head, B and C of N channels per group of heads; everything in float32.
//
//   ssd_step:         one token a sequence (decode steps), with the short convolution in front of it in the same kernel.
//   ssd_scan:         token by token (short portions).  The rows of S never mix, so 16 lanes share a value
//                     channel, each with a run of its N entries in registers.
//   ssd_chunk_scores, ssd_chunk_walk: long steps, in chunks of 64 tokens as matrix products (float32 matrix instructions:
//                     true 32-bit products and sums).  With l_t the sum of the chunk's log decays up to and with token t,
//                       y_t = exp(l_t) S C_t + sum_{s <= t} M_ts x_s + skip x_t,    M_ts = (C_t . B_s) exp(l_t - l_s) d_s
//                       S  <- exp(l_end) S + sum_s d_s exp(l_end - l_s) x_s B_s^T
//                     The first kernel makes every chunk's M (side by side, nothing depends on the state); the second walks
//                     a sequence's chunks with the state in accumulators, 16 value channels of a head a block.  The sums
//                     l are kept in float64 until their differences are taken: a chunk may decay by hundreds of e-folds,
//                     and neighbours' differences are small.
//   gated_group_norm: y * silu(z), each of `parts` equal parts of the row over its own root mean square, times a weight; in a
//                     decode step further blocks of the same launch move the convolution's state on.
//
// The state is kept [slot][head][value channel][state row], so that a lane's entries are contiguous.
#include "common.h"
#include "fmsamd.h"
#include "short_conv.h"

#define SSD_MAX_STATE 256
#define SSD_COLS 16  // value channels of a block of the token-by-token kernel

struct SsdArgs {
  const float* xbc;  // [T, ld]: x [H*P] | B [G*N] | C [G*N]
  long ld;
  const float* dt;  // [T, ld_dt]
  long ld_dt;
  const float *a_log, *dt_bias, *skip;  // [H]
  float* state;                         // [slots][H][P][N]
  float* y;                             // [T, H*P]
  const int *seq_starts, *seq_of_token, *slot_ids;
  int H, P, G, N;
};

template <int R>
__global__ void __launch_bounds__(256) ssd_scan_kernel(SsdArgs a) {
  const int b = blockIdx.x, h = blockIdx.y;
  const int t0 = a.seq_starts[b], t1 = a.seq_starts[b + 1];
  if (t0 >= t1 || a.seq_of_token[t0] < 0) return;
  const int slot = a.slot_ids[b];
  const int part = threadIdx.x & 15, p = blockIdx.z * SSD_COLS + (threadIdx.x >> 4);
  const int H = a.H, P = a.P, N = a.N, group = h / (H / a.G);
  const bool live = p < P;
  float* srow = a.state + (((size_t)slot * H + h) * P + (live ? p : 0)) * N + part * R;
  float S[R];
#pragma unroll
  for (int r = 0; r < R; ++r) S[r] = (live && part * R + r < N) ? srow[r] : 0.f;
  const float rate = -expf(a.a_log[h]), bias = a.dt_bias[h], skip = a.skip[h];
  for (int t = t0; t < t1; ++t) {
    const float* row = a.xbc + (size_t)t * a.ld;
    const float* Brow = row + (size_t)H * P + (size_t)group * N + part * R;
    const float* Crow = Brow + (size_t)a.G * N;
    const float x = live ? row[(size_t)h * P + p] : 0.f;
    const float d = softplus_f32(a.dt[(size_t)t * a.ld_dt + h] + bias);
    float Bv[R], Cv[R];
#pragma unroll
    for (int r = 0; r < R; ++r) {
      Bv[r] = part * R + r < N ? Brow[r] : 0.f;
      Cv[r] = part * R + r < N ? Crow[r] : 0.f;
    }
    const float decay = expf(rate * d), dx = d * x;
    float y = 0.f;
#pragma unroll
    for (int r = 0; r < R; ++r) {
      S[r] = fmaf(dx, Bv[r], decay * S[r]);
      y = fmaf(S[r], Cv[r], y);
    }
    y = row16_sum(y);
    if (live && part == 0) a.y[(size_t)t * H * P + (size_t)h * P + p] = fmaf(skip, x, y);
  }
  if (live) {
#pragma unroll
    for (int r = 0; r < R; ++r)
      if (part * R + r < N) srow[r] = S[r];
  }
}

static int ssd_check(const char* name, const SsdArgs& a, int n_seqs) {
  FMS_REQUIRE(n_seqs > 0 && a.H > 0 && a.P > 0 && a.G > 0 && a.H % a.G == 0 && a.N > 0 && a.N <= SSD_MAX_STATE,
              "%s: bad sizes heads=%d vdim=%d groups=%d state=%d", name, a.H, a.P, a.G, a.N);
  FMS_REQUIRE(a.ld >= (long)a.H * a.P + 2L * a.G * a.N && a.ld_dt >= a.H, "%s: rows too short", name);
  FMS_REQUIRE(a.H <= 65535 && ceil_div(a.P, SSD_COLS) <= 65535, "%s: too many heads or value channels for one launch", name);
  return 0;
}

extern "C" int fmsamd_ssd_scan(const float* xbc, long ld, const float* dt, long ld_dt, const float* a_log, const float* dt_bias,
                               const float* skip, float* state, float* y, const int* seq_starts, const int* seq_of_token,
                               const int* slot_ids, int n_seqs, int heads, int vdim, int groups, int n_state, hipStream_t stream) {
  if (n_seqs == 0) return 0;
  SsdArgs a{xbc, ld, dt, ld_dt, a_log, dt_bias, skip, state, y, seq_starts, seq_of_token, slot_ids, heads, vdim, groups, n_state};
  if (ssd_check("ssd_scan", a, n_seqs)) return -1;
  const dim3 grid(n_seqs, heads, ceil_div(vdim, SSD_COLS));
  if (n_state <= 16) ssd_scan_kernel<1><<<grid, 256, 0, stream>>>(a);
  else if (n_state <= 32) ssd_scan_kernel<2><<<grid, 256, 0, stream>>>(a);
  else if (n_state <= 64) ssd_scan_kernel<4><<<grid, 256, 0, stream>>>(a);
  else if (n_state <= 128) ssd_scan_kernel<8><<<grid, 256, 0, stream>>>(a);
  else ssd_scan_kernel<16><<<grid, 256, 0, stream>>>(a);
  FMS_LAUNCH_CHECK("ssd_scan");
  return 0;
}

// ---- long steps, in chunks -------------------------------------------------------------------------------------------------
#define SSD_CHUNK 64
#define SSD_HEADS 8  // heads of a block of ssd_chunk_scores, at most

// What the chunks of a step leave for the walk, by chunk slot and head: M [64][64], the weights of the tokens in the state
// d_s exp(l_end - l_s) [64], and exp(l_t) [64].  Chunk i of sequence b has the slot seq_starts[b] / 64 + b + i.
struct SsdChunks {
  float *m, *w, *e;
};
__device__ __forceinline__ int ssd_chunk_slot(int start, int b, int i) { return start / SSD_CHUNK + b + i; }

// Four entries n .. n + 3 of a row of B or C (zeros from N on).
template <bool VEC>
__device__ __forceinline__ f32x4 ssd_row4(const float* row, int n, int N) {
  if (VEC) return n < N ? *reinterpret_cast<const f32x4*>(row + n) : f32x4{0.f, 0.f, 0.f, 0.f};
  f32x4 v;
#pragma unroll
  for (int i = 0; i < 4; ++i) v[i] = n + i < N ? row[n + i] : 0.f;
  return v;
}

// The float32 product: lane (r = lane % 16, g = lane / 16) holds A[row r][k g] and B[k g][column r], and rows 4 g + i of
// column r of the result.  Which k a step takes is free as long as both operands agree: four steps take the k's
// 4 g + i, i = 0 .. 3, of sixteen, so that a lane's operands of four steps are four neighbours in memory.
#define SSD_MFMA(a, b, c) __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0)

template <bool VEC>
__global__ void __launch_bounds__(256) ssd_chunk_scores_kernel(SsdArgs a, SsdChunks out, int subsets) {
  __shared__ double ls[SSD_HEADS][SSD_CHUNK];
  __shared__ float ds[SSD_HEADS][SSD_CHUNK];
  const int b = blockIdx.y;
  const int start = a.seq_starts[b], t1 = a.seq_starts[b + 1];
  const int t0 = start + blockIdx.x * SSD_CHUNK;
  if (t0 >= t1 || a.seq_of_token[start] < 0) return;
  const int group = blockIdx.z / subsets, subset = blockIdx.z % subsets;
  const int per = a.H / a.G;
  const int h0 = group * per + subset * SSD_HEADS;
  const int nh = min(SSD_HEADS, per - subset * SSD_HEADS);
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, r = lane & 15, g = lane >> 4;
  const size_t slot = ssd_chunk_slot(start, b, blockIdx.x);
  const int last = t1 - 1;
  // decays: a lane a token, a wave a head
  for (int hh = wave; hh < nh; hh += 4) {
    const int h = h0 + hh, t = t0 + lane;
    float d = 0.f;  // past the sequence's end: a token that changes nothing
    if (t <= last) d = softplus_f32(a.dt[(size_t)t * a.ld_dt + h] + a.dt_bias[h]);
    double l = -(double)(expf(a.a_log[h]) * d);
#pragma unroll
    for (int off = 1; off < 64; off <<= 1) {
      const double o = __shfl_up(l, off, WAVE);
      if (lane >= off) l += o;
    }
    const double end = __shfl(l, 63, WAVE);
    ls[hh][lane] = l;
    ds[hh][lane] = d;
    out.w[(slot * a.H + h) * SSD_CHUNK + lane] = d * expf((float)(end - l));
    out.e[(slot * a.H + h) * SSD_CHUNK + lane] = expf((float)l);
  }
  // C_t . B_s for the wave's 16 tokens t and all tiles of s up to its own
  const size_t col_b = (size_t)a.H * a.P + (size_t)group * a.N, col_c = col_b + (size_t)a.G * a.N;
  const float* crow = a.xbc + (size_t)min(t0 + 16 * wave + r, last) * a.ld + col_c;
  const float* brow[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) brow[j] = a.xbc + (size_t)min(t0 + 16 * j + r, last) * a.ld + col_b;
  f32x4 cb[4];
#pragma unroll
  for (int j = 0; j < 4; ++j) cb[j] = f32x4{0.f, 0.f, 0.f, 0.f};
  for (int n0 = 0; n0 < a.N; n0 += 16) {
    const f32x4 c = ssd_row4<VEC>(crow, n0 + 4 * g, a.N);
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      if (j <= wave) {
        const f32x4 bv = ssd_row4<VEC>(brow[j], n0 + 4 * g, a.N);
#pragma unroll
        for (int i = 0; i < 4; ++i) cb[j] = SSD_MFMA(c[i], bv[i], cb[j]);
      }
    }
  }
  __syncthreads();
  for (int hh = 0; hh < nh; ++hh) {
    float* m = out.m + (slot * a.H + h0 + hh) * (SSD_CHUNK * SSD_CHUNK);
    double lt[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) lt[i] = ls[hh][16 * wave + 4 * g + i];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      if (j <= wave) {
        const int s = 16 * j + r;
        const double lsj = ls[hh][s];
        const float d = ds[hh][s];
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int t = 16 * wave + 4 * g + i;
          m[t * SSD_CHUNK + s] = s <= t ? cb[j][i] * expf((float)(lt[i] - lsj)) * d : 0.f;
        }
      }
    }
  }
}

// KT: tiles of 16 state rows a wave owns (N <= 64 KT)
template <int KT, bool VEC>
__global__ void __launch_bounds__(256) ssd_chunk_walk_kernel(SsdArgs a, SsdChunks in, int p_tiles, int n_seqs) {
  constexpr int NT = 4 * KT;
  __shared__ f32x4 states[2][NT * 64];  // the state as the chunk finds it: [tile][lane]
  // Blocks are dealt over the chip's eight dies in turn, each with a cache of its own: a run of neighbouring heads (which
  // share B and C, and a head's blocks its M) goes to one die.
  const int per_seq = a.H * p_tiles;
  const int b = blockIdx.x / per_seq;
  int id = blockIdx.x % per_seq;
  if (a.H % 8 == 0) id = (id % 8) * (per_seq / 8) + id / 8;
  const int h = id / p_tiles, p0 = (id % p_tiles) * 16;
  const int t0 = a.seq_starts[b], t1 = a.seq_starts[b + 1];
  if (t0 >= t1 || a.seq_of_token[t0] < 0) return;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, r = lane & 15, g = lane >> 4;
  const int N = a.N, P = a.P, last = t1 - 1;
  const int p = p0 + r;
  const bool live = p < P;
  const int group = h / (a.H / a.G);
  const size_t col_x = (size_t)h * P + (live ? p : 0);
  const size_t col_b = (size_t)a.H * P + (size_t)group * N, col_c = col_b + (size_t)a.G * N;
  float* srow = a.state + (((size_t)a.slot_ids[b] * a.H + h) * P + (live ? p : 0)) * N;
  const float skip = a.skip[h];

  f32x4 S[KT];  // state rows 16 (wave + 4 k) + 4 g + i of channel p
#pragma unroll
  for (int k = 0; k < KT; ++k) S[k] = ssd_row4<VEC>(srow, 16 * (wave + 4 * k) + 4 * g, live ? N : 0);

  struct Operands {
    f32x4 c[NT], m[4], w[4], e;
    float x[4][4], bb[KT][4][4], end;
  };
  auto load = [&](Operands& o, int chunk) {
    const int tc = t0 + chunk * SSD_CHUNK;
    const size_t slot = (size_t)ssd_chunk_slot(t0, b, chunk) * a.H + h;
    const float* crow = a.xbc + (size_t)min(tc + 16 * wave + r, last) * a.ld + col_c;
#pragma unroll
    for (int n = 0; n < NT; ++n) o.c[n] = ssd_row4<VEC>(crow, 16 * n + 4 * g, N);
    const float* m = in.m + slot * (SSD_CHUNK * SSD_CHUNK) + (16 * wave + r) * SSD_CHUNK + 4 * g;
    const float* w = in.w + slot * SSD_CHUNK + 4 * g;
    const float* e = in.e + slot * SSD_CHUNK;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      o.m[j] = *reinterpret_cast<const f32x4*>(m + (j <= wave ? 16 * j : 0));  // tiles above the diagonal are not there
      o.w[j] = *reinterpret_cast<const f32x4*>(w + 16 * j);
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const float* row = a.xbc + (size_t)min(tc + 16 * j + 4 * g + i, last) * a.ld;
        o.x[j][i] = row[col_x];
#pragma unroll
        for (int k = 0; k < KT; ++k) {
          const int n = 16 * (wave + 4 * k) + r;
          o.bb[k][j][i] = n < N ? row[col_b + n] : 0.f;
        }
      }
    }
    o.e = *reinterpret_cast<const f32x4*>(e + 16 * wave + 4 * g);
    o.end = e[SSD_CHUNK - 1];
  };
  auto work = [&](const Operands& o, int chunk) {
    f32x4* st = states[chunk & 1];  // the other buffer may still be read by a wave of the chunk before
#pragma unroll
    for (int k = 0; k < KT; ++k) st[(wave + 4 * k) * 64 + lane] = S[k];
    block_sync_lds();
    f32x4 y0 = f32x4{0.f, 0.f, 0.f, 0.f}, y1 = y0;
#pragma unroll
    for (int n = 0; n < NT; n += 2) {
      const f32x4 s0 = st[n * 64 + lane], s1 = st[(n + 1) * 64 + lane];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        y0 = SSD_MFMA(o.c[n][i], s0[i], y0);
        y1 = SSD_MFMA(o.c[n + 1][i], s1[i], y1);
      }
    }
    f32x4 y = (y0 + y1) * o.e;
    f32x4 xt = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      if (j <= wave) {  // uniform over the wave
#pragma unroll
        for (int i = 0; i < 4; ++i) y = SSD_MFMA(o.m[j][i], o.x[j][i], y);
      }
      if (j == wave) xt = f32x4{o.x[j][0], o.x[j][1], o.x[j][2], o.x[j][3]};
    }
#pragma unroll
    for (int k = 0; k < KT; ++k) S[k] *= o.end;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const float xw = o.x[j][i] * o.w[j][i];
#pragma unroll
        for (int k = 0; k < KT; ++k) S[k] = SSD_MFMA(o.bb[k][j][i], xw, S[k]);
      }
    }
    const int t = t0 + chunk * SSD_CHUNK + 16 * wave + 4 * g;
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (live && t + i <= last) a.y[(size_t)(t + i) * a.H * P + (size_t)h * P + p] = fmaf(skip, xt[i], y[i]);
  };
  // the next chunk's operands are asked for before this one is worked on
  const int chunks = (t1 - t0 + SSD_CHUNK - 1) / SSD_CHUNK;
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
      const int n = 16 * (wave + 4 * k) + 4 * g;
      if (VEC) {
        if (n < N) *reinterpret_cast<f32x4*>(srow + n) = S[k];
      } else {
#pragma unroll
        for (int i = 0; i < 4; ++i)
          if (n + i < N) srow[n + i] = S[k][i];
      }
    }
  }
}

extern "C" long fmsamd_ssd_chunk_workspace(int n_tokens, int n_seqs, int heads) {
  const long slots = n_tokens / SSD_CHUNK + n_seqs + 1;
  return slots * heads * (SSD_CHUNK * SSD_CHUNK + 2 * SSD_CHUNK) * (long)sizeof(float);
}

extern "C" int fmsamd_ssd_chunked(const float* xbc, long ld, const float* dt, long ld_dt, const float* a_log, const float* dt_bias,
                                  const float* skip, float* state, float* y, const int* seq_starts, const int* seq_of_token,
                                  const int* slot_ids, int n_seqs, int heads, int vdim, int groups, int n_state, int n_tokens, int longest,
                                  float* workspace, long workspace_bytes, hipStream_t stream) {
  if (n_seqs == 0 || n_tokens == 0) return 0;
  SsdArgs a{xbc, ld, dt, ld_dt, a_log, dt_bias, skip, state, y, seq_starts, seq_of_token, slot_ids, heads, vdim, groups, n_state};
  if (ssd_check("ssd_chunked", a, n_seqs)) return -1;
  FMS_REQUIRE(longest > 0 && longest <= n_tokens, "ssd_chunked: a longest sequence of %d in %d tokens", longest, n_tokens);
  FMS_REQUIRE(workspace != nullptr && workspace_bytes >= fmsamd_ssd_chunk_workspace(n_tokens, n_seqs, heads) && (uintptr_t)workspace % 16 == 0,
              "ssd_chunked: the workspace is too small");
  const long slots = n_tokens / SSD_CHUNK + n_seqs + 1;
  SsdChunks c{workspace, workspace + slots * heads * SSD_CHUNK * SSD_CHUNK,
              workspace + slots * heads * (SSD_CHUNK * SSD_CHUNK + SSD_CHUNK)};
  const int subsets = ceil_div(heads / groups, SSD_HEADS);
  FMS_REQUIRE(n_seqs <= 65535 && (long)groups * subsets <= 65535, "ssd_chunked: too many sequences or groups for one launch");
  const int p_tiles = ceil_div(vdim, 16);
  const long blocks = (long)n_seqs * heads * p_tiles;
  FMS_REQUIRE(blocks < (1L << 31), "ssd_chunked: too many blocks");
  const bool vec = n_state % 4 == 0 && ((long)heads * vdim) % 4 == 0 && ld % 4 == 0 && (uintptr_t)xbc % 16 == 0 && (uintptr_t)state % 16 == 0;
  const dim3 grid(ceil_div(longest, SSD_CHUNK), n_seqs, groups * subsets);
  if (vec) ssd_chunk_scores_kernel<true><<<grid, 256, 0, stream>>>(a, c, subsets);
  else ssd_chunk_scores_kernel<false><<<grid, 256, 0, stream>>>(a, c, subsets);
  FMS_LAUNCH_CHECK("ssd_chunk_scores");
#define FMS_SSD_WALK(KT)                                                                                       \
  do {                                                                                                         \
    if (vec) ssd_chunk_walk_kernel<KT, true><<<(unsigned)blocks, 256, 0, stream>>>(a, c, p_tiles, n_seqs);     \
    else ssd_chunk_walk_kernel<KT, false><<<(unsigned)blocks, 256, 0, stream>>>(a, c, p_tiles, n_seqs);        \
  } while (0)
  if (n_state <= 64) FMS_SSD_WALK(1);
  else if (n_state <= 128) FMS_SSD_WALK(2);
  else FMS_SSD_WALK(4);
#undef FMS_SSD_WALK
  FMS_LAUNCH_CHECK("ssd_chunk_walk");
  return 0;
}

// ---- decode steps: one token a sequence ------------------------------------------------------------------------------------
// The short convolution, its silu, the step sizes and the recurrence of a (sequence, head) in one kernel: a block forms its
// own 64 value channels and its group's B and C from the projection and the convolution's state (which it only reads: the
// other heads of the group read it too; conv_move, which runs with the next kernel, moves it on), while its rows of S are on
// their way.  A row of S is shared by 16 lanes, four neighbouring entries a load.
struct SsdStep {
  const float* proj;  // [T, ld]: convolved channels at col_x, step sizes at col_dt
  long ld;
  int col_x, col_dt;
  const void *conv_w, *conv_b;  // [C, taps], [C]
  int taps;
  const float* conv_state;  // [slots][taps - 1][C]
  const float *a_log, *dt_bias, *skip;
  float *state, *y;
  const int *seq_starts, *seq_of_token, *slot_ids;
  int H, P, G, N;
};
#define SSD_STEP_ROWS 64  // value channels of a block

template <int K4, bool VEC, typename W>
__global__ void __launch_bounds__(256) ssd_step_kernel(SsdStep a) {
  constexpr int TILES = SSD_STEP_ROWS / 16;
  __shared__ __attribute__((aligned(16))) float u[SSD_STEP_ROWS + 2 * 64 * K4];  // x | B | C, each of B and C padded to 64 K4 entries
  const int h = blockIdx.x, b = blockIdx.y;
  const int t = uniform_load(a.seq_starts + b);
  if (uniform_load(a.seq_of_token + t) < 0) return;
  const int slot = uniform_load(a.slot_ids + b);
  const int H = a.H, P = a.P, N = a.N, group = h / (H / a.G), p0 = blockIdx.z * SSD_STEP_ROWS;
  const int C = H * P + 2 * a.G * N;
  const int part = threadIdx.x & 15, row = threadIdx.x >> 4;
  float* const st = a.state + (((size_t)slot * H + h) * P + p0) * N;
  f32x4 S[TILES][K4];
#pragma unroll
  for (int i = 0; i < TILES; ++i) {
    const int p = i * 16 + row;
#pragma unroll
    for (int k = 0; k < K4; ++k) S[i][k] = ssd_row4<VEC>(st + (size_t)(p0 + p < P ? p : 0) * N, 64 * k + 4 * part, p0 + p < P ? N : 0);
  }
  const float dt = a.proj[(size_t)t * a.ld + a.col_dt + h] + a.dt_bias[h];
  const float rate = -expf(a.a_log[h]), skip = a.skip[h];
  // the convolved channels: 64 of x, then B, then C
  const float* now = a.proj + (size_t)t * a.ld + a.col_x;
  const float* old = a.conv_state + (size_t)slot * (a.taps - 1) * C;
  const W* cw = (const W*)a.conv_w;
  const W* cbias = (const W*)a.conv_b;
  for (int i = threadIdx.x; i < SSD_STEP_ROWS + 2 * 64 * K4; i += 256) {
    int c = -1;
    if (i < SSD_STEP_ROWS) {
      if (p0 + i < P) c = h * P + p0 + i;
    } else {
      const int j = (i - SSD_STEP_ROWS) % (64 * K4), which = (i - SSD_STEP_ROWS) / (64 * K4);
      if (j < N) c = H * P + (which * a.G + group) * N + j;
    }
    float v = 0.f;
    if (c >= 0) {
      float x[CONV_MAX_TAPS], w[CONV_MAX_TAPS];
#pragma unroll
      for (int j = 0; j < CONV_MAX_TAPS; ++j) {
        x[j] = w[j] = 0.f;
        if (j < a.taps) {
          x[j] = j == a.taps - 1 ? now[c] : old[(size_t)j * C + c];
          w[j] = to_f32(cw[(size_t)c * a.taps + j]);
        }
      }
      float acc = to_f32(cbias[c]);
#pragma unroll
      for (int j = 0; j < CONV_MAX_TAPS; ++j) acc = fmaf(w[j], x[j], acc);
      v = acc / (1.f + expf(-acc));
    }
    u[i] = v;
  }
  __syncthreads();
  const float d = softplus_f32(dt), decay = expf(rate * d);
  f32x4 Bv[K4], Cv[K4];
#pragma unroll
  for (int k = 0; k < K4; ++k) {
    Bv[k] = *reinterpret_cast<const f32x4*>(u + SSD_STEP_ROWS + 64 * k + 4 * part);
    Cv[k] = *reinterpret_cast<const f32x4*>(u + SSD_STEP_ROWS + 64 * K4 + 64 * k + 4 * part);
  }
#pragma unroll
  for (int i = 0; i < TILES; ++i) {
    const int p = i * 16 + row;
    const float x = u[p], dx = d * x;
    float y = 0.f;
#pragma unroll
    for (int k = 0; k < K4; ++k) {
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        S[i][k][e] = fmaf(dx, Bv[k][e], decay * S[i][k][e]);
        y = fmaf(S[i][k][e], Cv[k][e], y);
      }
    }
    y = row16_sum(y);
    if (p0 + p < P) {
      if (part == 0) a.y[(size_t)t * H * P + (size_t)h * P + p0 + p] = fmaf(skip, x, y);
#pragma unroll
      for (int k = 0; k < K4; ++k) {
        const int n = 64 * k + 4 * part;
        float* dst = st + (size_t)p * N + n;
        if (VEC) {
          if (n < N) *reinterpret_cast<f32x4*>(dst) = S[i][k];
        } else {
#pragma unroll
          for (int e = 0; e < 4; ++e)
            if (n + e < N) dst[e] = S[i][k][e];
        }
      }
    }
  }
}

extern "C" int fmsamd_ssd_step(const float* proj, long ld, int col_x, int col_dt, const void* conv_w, const void* conv_b, int weight_dtype,
                               int taps, const float* conv_state, const float* a_log, const float* dt_bias, const float* skip, float* state,
                               float* y, const int* seq_starts, const int* seq_of_token, const int* slot_ids, int n_seqs, int heads,
                               int vdim, int groups, int n_state, hipStream_t stream) {
  if (n_seqs == 0) return 0;
  SsdStep a{proj, ld, col_x, col_dt, conv_w, conv_b, taps, conv_state, a_log, dt_bias, skip, state, y, seq_starts, seq_of_token, slot_ids,
            heads, vdim, groups, n_state};
  FMS_REQUIRE(n_seqs > 0 && n_seqs <= 65535 && heads > 0 && vdim > 0 && groups > 0 && heads % groups == 0 && n_state > 0 && n_state <= SSD_MAX_STATE,
              "ssd_step: bad sizes heads=%d vdim=%d groups=%d state=%d", heads, vdim, groups, n_state);
  const long C = (long)heads * vdim + 2L * groups * n_state;
  FMS_REQUIRE(col_x >= 0 && col_x + C <= ld && col_dt >= 0 && col_dt + heads <= ld, "ssd_step: the rows do not hold the columns asked for");
  FMS_REQUIRE(taps >= 1 && taps <= CONV_MAX_TAPS && (taps == 1 || conv_state != nullptr), "ssd_step: %d taps (1 to %d, with a state)", taps, CONV_MAX_TAPS);
  FMS_REQUIRE(ceil_div(vdim, SSD_STEP_ROWS) <= 65535, "ssd_step: too many value channels");
  const bool vec = n_state % 4 == 0 && (uintptr_t)state % 16 == 0;
  const dim3 grid(heads, n_seqs, ceil_div(vdim, SSD_STEP_ROWS));
#define FMS_STEP(K4)                                                                      \
  do {                                                                                    \
    if (weight_dtype == FMS_F32) {                                                        \
      if (vec) ssd_step_kernel<K4, true, float><<<grid, 256, 0, stream>>>(a);             \
      else ssd_step_kernel<K4, false, float><<<grid, 256, 0, stream>>>(a);                \
    } else {                                                                              \
      if (vec) ssd_step_kernel<K4, true, bf16><<<grid, 256, 0, stream>>>(a);              \
      else ssd_step_kernel<K4, false, bf16><<<grid, 256, 0, stream>>>(a);                 \
    }                                                                                     \
  } while (0)
  FMS_REQUIRE(weight_dtype == FMS_F32 || weight_dtype == FMS_BF16, "ssd_step: unknown dtype %d", weight_dtype);
  if (n_state <= 64) FMS_STEP(1);
  else if (n_state <= 128) FMS_STEP(2);
  else FMS_STEP(4);
#undef FMS_STEP
  FMS_LAUNCH_CHECK("ssd_step");
  return 0;
}

// ---- the gated norm --------------------------------------------------------------------------------------------------------
// A convolution's state to be moved on by one token a sequence (a decode step), by blocks of their own beside the norm's.
struct ConvMove {
  const float* x;  // float32 rows ld apart, at the first convolved channel
  long ld;
  int channels, taps;
  float* state;  // [slots][taps - 1][channels]
  const int* slot_ids;
};
__device__ __forceinline__ void conv_move(const ConvMove& m, const int* seq_of_token, int t, int c) {
  const int seq = seq_of_token[t];
  if (seq < 0 || c >= m.channels) return;
  float* st = m.state + (size_t)m.slot_ids[seq] * (m.taps - 1) * m.channels + c;
  float v[CONV_MAX_TAPS];
#pragma unroll
  for (int j = 0; j < CONV_MAX_TAPS - 1; ++j)
    if (j < m.taps - 1) v[j] = j + 1 < m.taps - 1 ? st[(size_t)(j + 1) * m.channels] : m.x[(size_t)t * m.ld + c];
#pragma unroll
  for (int j = 0; j < CONV_MAX_TAPS - 1; ++j)
    if (j < m.taps - 1) st[(size_t)j * m.channels] = v[j];
}

__device__ __forceinline__ float gated(float y, float z) { return y * (z / (1.f + expf(-z))); }

// A wave per (token, part), for parts of at most 1024 channels: the part's gated values wait in registers, four neighbours a
// load, and no wave waits for another.  Blocks from norm_blocks on move the convolution's state.
template <typename T, typename W>
__global__ void __launch_bounds__(256)
    gated_group_norm_wave_kernel(const float* __restrict__ y, const float* __restrict__ z, long ldz, const W* __restrict__ weight, float eps,
                                 T* __restrict__ out, const int* __restrict__ seq_of_token, int n_tokens, int cols, int size, int norm_blocks,
                                 ConvMove move, int move_blocks) {
  if ((int)blockIdx.x >= norm_blocks) {
    const int i = blockIdx.x - norm_blocks;
    conv_move(move, seq_of_token, i / move_blocks, (i % move_blocks) * 256 + threadIdx.x);
    return;
  }
  const int parts = cols / size;
  const long item = (long)blockIdx.x * 4 + (threadIdx.x >> 6);
  const int lane = threadIdx.x & 63;
  const int t = (int)(item / parts), part = (int)(item % parts);
  if (t >= n_tokens || seq_of_token[t] < 0) return;
  const float* yr = y + (size_t)t * cols + (size_t)part * size;
  const float* zr = z + (size_t)t * ldz + (size_t)part * size;
  const W* wr = weight + (size_t)part * size;
  T* o = out + (size_t)t * cols + (size_t)part * size;
  f32x4 v[4];
  float s = 0.f;
#pragma unroll
  for (int n = 0; n < 4; ++n) {
    const int i = (n * 64 + lane) * 4;
    v[n] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (i < size) {
      const f32x4 yv = *reinterpret_cast<const f32x4*>(yr + i), zv = *reinterpret_cast<const f32x4*>(zr + i);
#pragma unroll
      for (int e = 0; e < 4; ++e) v[n][e] = gated(yv[e], zv[e]), s = fmaf(v[n][e], v[n][e], s);
    }
  }
  const float inv = 1.f / sqrtf(wave_sum(s) / (float)size + eps);
#pragma unroll
  for (int n = 0; n < 4; ++n) {
    const int i = (n * 64 + lane) * 4;
    if (i < size) {
      T r[4];
#pragma unroll
      for (int e = 0; e < 4; ++e) r[e] = from_f32<T>(v[n][e] * inv * to_f32(wr[i + e]));
      if constexpr (sizeof(T) == 2) *reinterpret_cast<bf16x4*>(o + i) = bf16x4{r[0], r[1], r[2], r[3]};
      else *reinterpret_cast<f32x4*>(o + i) = f32x4{r[0], r[1], r[2], r[3]};
    }
  }
}

// A block per (token, part); the part's gated values wait in registers (up to 16 a thread, the rest is formed again).
template <typename T, typename W>
__global__ void __launch_bounds__(1024)
    gated_group_norm_kernel(const float* __restrict__ y, const float* __restrict__ z, long ldz, const W* __restrict__ weight, float eps,
                            T* __restrict__ out, const int* __restrict__ seq_of_token, int cols, int size, int norm_blocks, ConvMove move,
                            int move_blocks) {
  __shared__ float scratch[17];
  constexpr int KEEP = 16;
  if ((int)blockIdx.x >= norm_blocks) {
    const int i = blockIdx.x - norm_blocks;
    const int c = (i % move_blocks) * 256;
    for (int k = threadIdx.x; k < 256; k += blockDim.x) conv_move(move, seq_of_token, i / move_blocks, c + k);
    return;
  }
  const int parts = cols / size;
  const int t = blockIdx.x / parts, c0 = (blockIdx.x % parts) * size;
  if (seq_of_token[t] < 0) return;
  const float* yr = y + (size_t)t * cols + c0;
  const float* zr = z + (size_t)t * ldz + c0;
  const W* wr = weight + c0;
  T* o = out + (size_t)t * cols + c0;
  float keep[KEEP], s = 0.f;
#pragma unroll
  for (int n = 0; n < KEEP; ++n) {
    const int i = threadIdx.x + n * blockDim.x;
    keep[n] = i < size ? gated(yr[i], zr[i]) : 0.f;
    s = fmaf(keep[n], keep[n], s);
  }
  for (int i = threadIdx.x + KEEP * blockDim.x; i < size; i += blockDim.x) {
    const float v = gated(yr[i], zr[i]);
    s = fmaf(v, v, s);
  }
  const float inv = 1.f / sqrtf(block_sum(s, scratch) / (float)size + eps);
#pragma unroll
  for (int n = 0; n < KEEP; ++n) {
    const int i = threadIdx.x + n * blockDim.x;
    if (i < size) o[i] = from_f32<T>(keep[n] * inv * to_f32(wr[i]));
  }
  for (int i = threadIdx.x + KEEP * blockDim.x; i < size; i += blockDim.x) o[i] = from_f32<T>(gated(yr[i], zr[i]) * inv * to_f32(wr[i]));
}

extern "C" int fmsamd_gated_group_norm(const float* y, const float* z, long ldz, const void* weight, int weight_dtype, int parts, float eps,
                                       void* out, int out_dtype, const int* seq_of_token, int n_tokens, int cols, const float* conv_x,
                                       long ld_conv, int channels, int taps, float* conv_state, const int* slot_ids, hipStream_t stream) {
  if (n_tokens == 0) return 0;
  FMS_REQUIRE(n_tokens > 0 && cols > 0 && parts > 0 && cols % parts == 0 && ldz >= cols, "gated_group_norm: %d parts of %d channels", parts, cols);
  const int size = cols / parts;
  ConvMove move{conv_x, ld_conv, channels, taps, conv_state, slot_ids};
  int move_blocks = 0;  // a token's
  if (conv_x != nullptr) {
    FMS_REQUIRE(taps >= 2 && taps <= CONV_MAX_TAPS && channels > 0 && ld_conv >= channels && conv_state != nullptr && slot_ids != nullptr,
                "gated_group_norm: a state of %d taps over %d channels", taps, channels);
    move_blocks = ceil_div(channels, 256);
  }
  const bool by_waves = size <= 1024 && size % 4 == 0 && ldz % 4 == 0 && (((uintptr_t)y | (uintptr_t)z | (uintptr_t)out) & 15) == 0;
  const long norm_blocks = by_waves ? ceil_div((long)n_tokens * parts, 4) : (long)n_tokens * parts;
  const long blocks = norm_blocks + (long)n_tokens * move_blocks;
  FMS_REQUIRE(blocks < (1L << 31), "gated_group_norm: too many blocks");
  const int threads = size >= 2048 ? 512 : (size >= 512 ? 256 : 64);
#define FMS_GGN(T, W)                                                                                                                   \
  do {                                                                                                                                  \
    if (by_waves)                                                                                                                       \
      gated_group_norm_wave_kernel<T, W><<<(unsigned)blocks, 256, 0, stream>>>(y, z, ldz, (const W*)weight, eps, (T*)out, seq_of_token, \
                                                                               n_tokens, cols, size, (int)norm_blocks, move, move_blocks); \
    else                                                                                                                                \
      gated_group_norm_kernel<T, W><<<(unsigned)blocks, threads, 0, stream>>>(y, z, ldz, (const W*)weight, eps, (T*)out, seq_of_token,  \
                                                                              cols, size, (int)norm_blocks, move, move_blocks);         \
  } while (0)
  if (out_dtype == FMS_F32 && weight_dtype == FMS_F32) FMS_GGN(float, float);
  else if (out_dtype == FMS_BF16 && weight_dtype == FMS_F32) FMS_GGN(bf16, float);
  else if (out_dtype == FMS_BF16 && weight_dtype == FMS_BF16) FMS_GGN(bf16, bf16);
  else if (out_dtype == FMS_F32 && weight_dtype == FMS_BF16) FMS_GGN(float, bf16);
  else FMS_REQUIRE(false, "gated_group_norm: unknown dtypes %d, %d", out_dtype, weight_dtype);
#undef FMS_GGN
  FMS_LAUNCH_CHECK("gated_group_norm");
  return 0;
}
