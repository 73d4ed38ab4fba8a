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

// ---- matrix-core kernels: bfloat16 storage, float32 scores, softmax and sums ---------------------------------------------
// Both compute S^T = K Q^T (rows: keys, columns: queries or heads) over the row of all kv heads' keys, so that the
// probabilities come out of the accumulator in the operand layout of O^T = V^T P^T.  Scores live in the base-2 domain
// (scale2 = scale * log2(e)).
#define TALK_LOG2E 1.4426950408889634f
#define TALK_EMPTY -1e30f
#define TALK_PAD 8   // elements between LDS rows, beyond their length
#define TALK_KEYS 32 // keys of a tile

__device__ __forceinline__ bf16x8 talk_load8(const bf16* p) { return *reinterpret_cast<const bf16x8*>(p); }
// maxima as single instructions: the scores come out of the matrix unit and are never signalling NaNs
__device__ __forceinline__ float talk_max2(float a, float b) {
  float r;
  asm("v_max_f32 %0, %1, %2" : "=v"(r) : "v"(a), "v"(b));
  return r;
}
__device__ __forceinline__ float talk_max3(float a, float b, float c) {
  float r;
  asm("v_max3_f32 %0, %1, %2, %3" : "=v"(r) : "v"(a), "v"(b), "v"(c));
  return r;
}

struct TalkArgs {
  const bf16* q;
  long q_stride;
  bf16* out;
  long out_stride;
  const int *positions, *seq_of_token, *block_table;
  int table_stride;
  const bf16 *k_cache, *v_cache;
  const float *talk, *sink;
  int n_tokens, nheads, kvheads, dim, vdim;
  float scale;
  int window;
};

__device__ __forceinline__ int talk_first_key(int pos, int window) { return (window > 0 && pos - window + 1 > 0) ? pos - window + 1 : 0; }

// Eight entries of the mixed query of a head: kv head c, entries d .. d + 7 of its query heads summed with the head's row of the
// mixing matrix.  The heads' pieces are asked for four at a time.
__device__ __forceinline__ bf16x8 talk_mixed_query(const bf16* qrow, const float* mix, int c, int d, int per, int dim) {
  float s[8];
#pragma unroll
  for (int e = 0; e < 8; ++e) s[e] = 0.f;
  const bf16* src = qrow + (size_t)c * per * dim + d;
  for (int i0 = 0; i0 < per; i0 += 4) {
    bf16x8 v[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = talk_load8(src + (size_t)(i0 + i < per ? i0 + i : 0) * dim);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const float w = i0 + i < per ? mix[c * per + i0 + i] : 0.f;
#pragma unroll
      for (int e = 0; e < 8; ++e) s[e] = fmaf(w, (float)v[i][e], s[e]);
    }
  }
  return bf16x8{(bf16)s[0], (bf16)s[1], (bf16)s[2], (bf16)s[3], (bf16)s[4], (bf16)s[5], (bf16)s[6], (bf16)s[7]};
}

// Prompts.  A block has four units: `hb` heads of one kv head times 4 / hb runs of 32 consecutive query tokens of one
// sequence.  A unit is one head and 32 queries (one tile column of the 32x32x16 product) and has two waves, which split the
// entries of the mixed queries (a query's mixed row is as long as all kv heads' keys together, and half of it leaves a wave
// room to be one of two on its SIMD) and the keys behind them: a wave multiplies its half of every key row, hands its sums for
// the other's 16 keys of the tile over through LDS, and runs softmax and second product over its own 16; at the end the
// two waves' results are joined.  (Where the rows are longest, a wave's registers do not hold the accumulators of all value
// channels: there both waves take all 32 keys, and the value channels are split.)  Tiles of 32 keys (all kv heads' keys, and the values of the block's kv head) go through LDS: the
// keys are free as soon as the scores are formed, so the next tile's are written while this one's softmax and second product
// run, and the tile after that is on its way from memory.
//
// Which key sits in which row of the score tile is free: rows are dealt so that a lane's 16 scores are the keys 8 half ..
// 8 half + 7 and 16 + 8 half .. 16 + 8 half + 7, each eight the operand of one step of the second product.
#define TALK_UNITS 4
#define TALK_NOWHERE 0xffff0000u
#define TALK_PREFILL_THREADS (TALK_UNITS * 2 * WAVE)

template <int KC, int DT>
struct TalkPrefillLds {
  static constexpr int KS = KC * 16 + TALK_PAD;     // row stride of the keys [32][KS]
  static constexpr int VS = TALK_KEYS + TALK_PAD;   // row stride of the transposed values [DT * 32][VS]
  static constexpr int K_ELEMS = TALK_KEYS * KS, V_ELEMS = DT * 32 * VS;
  static constexpr bool SPLIT_VALUES = KC > 32 && DT > 2;
  static constexpr int OWN = SPLIT_VALUES ? 16 : 8;  // scores of a tile that a lane runs the softmax over
  static constexpr int EXCHANGE = TALK_UNITS * 2 * WAVE * OWN;  // float32: what every wave hands over
  static constexpr int BYTES = (K_ELEMS + 2 * V_ELEMS) * 2 + EXCHANGE * 4;
};

template <int KC, int DT>
__global__ void __launch_bounds__(TALK_PREFILL_THREADS) __attribute__((amdgpu_waves_per_eu(2, 2)))
    talking_prefill_kernel(TalkArgs a, const int* __restrict__ qblock_start, const int* __restrict__ qblock_len, int n_qblocks, int hb) {
  typedef TalkPrefillLds<KC, DT> L;
  constexpr int KH = KC / 2;  // a wave's share of the key entries, in steps of 16
  constexpr bool SPLIT_VALUES = L::SPLIT_VALUES;
  constexpr int OWN = L::OWN, DA = SPLIT_VALUES ? (DT + 1) / 2 : DT;  // DA: tiles of 32 value channels of a wave
  // The longest rows leave registers for half a tile of keys on its way: one half is under way while the scores are formed,
  // the other while softmax and second product run.
  constexpr bool HALVES = KC > 32;
  constexpr int KW = KC * 16, KS = L::KS, VS = L::VS;
  constexpr int KCH = TALK_KEYS * KW / 8 / TALK_PREFILL_THREADS;                                          // 16-byte pieces a thread
  constexpr int VCH = (DT * 32 * TALK_KEYS / 8 + TALK_PREFILL_THREADS - 1) / TALK_PREFILL_THREADS;  // moves per tile
  extern __shared__ __attribute__((aligned(16))) unsigned char talk_lds[];
  bf16* const ks = reinterpret_cast<bf16*>(talk_lds);
  bf16* const vs = ks + L::K_ELEMS;  // two of them, in turn
  f32x4* const exchange = reinterpret_cast<f32x4*>(vs + 2 * L::V_ELEMS);  // [wave][OWN / 4][lane]

  // Blocks with the most keys (a causal step's last) are handed out first.  Workgroups go to the chip's eight dies in turn,
  // each with a cache of its own: runs of four query blocks, whose windows overlap, with all their heads go to one die.
  const int per = a.nheads / a.kvheads, tiles = per / hb, per_qb = a.kvheads * tiles;
  int id = blockIdx.x;
  const int run = 4 * per_qb, whole = n_qblocks / 32 * 8 * run;  // blocks of whole rounds over the dies
  if (id < whole) id = ((id / 8 / run) * 8 + id % 8) * run + (id / 8) % run;
  const int qb = n_qblocks - 1 - id / per_qb;
  const int y = id % per_qb;
  const int kh = y / tiles;
  const int wave = threadIdx.x / WAVE, lane = threadIdx.x & (WAVE - 1);
  const int unit = wave >> 1, side = wave & 1;
  const int j = lane & 31, half = lane >> 5;
  const int h = kh * per + (y % tiles) * hb + unit % hb;
  const int t_begin = qblock_start[qb], t_end = t_begin + qblock_len[qb];
  const int seq = a.seq_of_token[t_begin];
  if (seq < 0) return;  // whole block: uniform
  const int* bt = a.block_table + (size_t)seq * a.table_stride;
  const size_t page_elems = (size_t)a.kvheads * PAGE_TOKENS * a.dim, vpage_elems = (size_t)a.kvheads * PAGE_TOKENS * a.vdim;

  // this unit's queries
  const int t0 = t_begin + (unit / hb) * 32;
  const bool has_work = t0 < t_end;
  const int t = t0 + j;
  const bool valid = t < t_end;
  const int row = a.kvheads * a.dim;  // entries of a key row
  // the mixed queries of one unit after the other pass through the keys' place in LDS: all threads form them, the unit's
  // waves take their halves.  (Their padding leaves zeros behind the keys' entries, which are multiplied by zeros later.)
  bf16x8 qreg[KH];
  float* const mix = reinterpret_cast<float*>(exchange);  // the heads' rows of the mixing matrix
  for (int i = threadIdx.x; i < hb * a.nheads; i += TALK_PREFILL_THREADS)
    mix[i] = a.talk[(size_t)(kh * per + (y % tiles) * hb) * a.nheads + i];
  // a thread's pieces share their entries k: a row has a power of two of pieces, or (384) 48, and tokens are 512 / that apart
  const int uk = (threadIdx.x % (KW / 8)) * 8, uc = uk < row ? uk / a.dim : 0, ud = uk - uc * a.dim;
  __syncthreads();
  for (int u = 0; u < TALK_UNITS; ++u) {
    const int ut = t_begin + (u / hb) * 32;
    for (int tok = threadIdx.x / (KW / 8); tok < 32; tok += TALK_PREFILL_THREADS / (KW / 8)) {
      if (KW == 384 && threadIdx.x >= TALK_PREFILL_THREADS / (KW / 8) * (KW / 8)) break;  // 480 of the threads have a piece
      bf16x8 v = {0, 0, 0, 0, 0, 0, 0, 0};
      if (ut + tok < t_end && uk < row)
        v = talk_mixed_query(a.q + (size_t)(ut + tok) * a.q_stride, mix + (u % hb) * a.nheads, uc, ud, per, a.dim);
      *reinterpret_cast<bf16x8*>(ks + tok * KS + uk) = v;
    }
    __syncthreads();
    if (u == unit) {
#pragma unroll
      for (int c = 0; c < KH; ++c) qreg[c] = talk_load8(ks + j * KS + (side * KH + c) * 16 + half * 8);
    }
    __syncthreads();
  }
  const int qpos = valid ? a.positions[t] : -1;
  const int qlo = valid ? talk_first_key(qpos, a.window) : 0;
  int wave_hi = -1, wave_lo = 0, full_hi = -1, full_lo = 0;  // keys some / every column of the unit sees
  if (has_work) {
    const int t_last = (t0 + 32 < t_end ? t0 + 32 : t_end) - 1;
    wave_hi = a.positions[t_last];
    full_hi = a.positions[t0];
    wave_lo = talk_first_key(full_hi, a.window);
    full_lo = talk_first_key(wave_hi, a.window);
  }
  const int tile_first = talk_first_key(a.positions[t_begin], a.window) / TALK_KEYS;
  const int tile_last = a.positions[t_end - 1] / TALK_KEYS;

  // where a thread's pieces of a tile lie in the page and in LDS (the same for every tile), in pieces of eight entries: the
  // place in LDS in the upper 16 bits (TALK_NOWHERE: the padding has no piece), the one in the page in the lower
  unsigned k_at[KCH];
  const int d8 = a.dim / 8;
#pragma unroll
  for (int n = 0; n < KCH; ++n) {
    const int id = threadIdx.x + n * TALK_PREFILL_THREADS;
    const int c = id / (TALK_KEYS * d8), rest = id - c * (TALK_KEYS * d8);
    const int tok = rest / d8, d = rest - tok * d8;
    const bool there = c < a.kvheads;
    k_at[n] = there ? (unsigned)(tok * (KS / 8) + c * d8 + d) << 16 | (unsigned)((c * PAGE_TOKENS + tok) * d8 + d) : TALK_NOWHERE;
  }
  const int v_pieces = a.vdim * (TALK_KEYS / 8);
  constexpr int KP = HALVES ? KCH / 2 : KCH;
  bf16x8 kbuf[KP], vbuf[VCH];
  // the pieces of a tile's keys from n0 on (and, with the first of them, its values) into registers, and on into LDS
  auto fetch = [&](int tile, int n0) {
    const int key0 = tile * TALK_KEYS;
    const size_t phys = readable_page(uniform_load(bt + key0 / PAGE_TOKENS));
    const int in_page = key0 % PAGE_TOKENS;
    const bf16* kp = a.k_cache + phys * page_elems + (size_t)in_page * a.dim;
    const bf16* vp = a.v_cache + phys * vpage_elems + (size_t)kh * a.vdim * PAGE_TOKENS + in_page;
#pragma unroll
    for (int n = 0; n < KP; ++n) kbuf[n] = talk_load8(kp + (size_t)(k_at[HALVES && n0 ? n + KCH - KP : n] & 0xffffu) * 8);
    if (n0) return;
#pragma unroll
    for (int n = 0; n < VCH; ++n) {
      const int id = threadIdx.x + n * TALK_PREFILL_THREADS;
      vbuf[n] = talk_load8(vp + (id < v_pieces ? (size_t)(id / (TALK_KEYS / 8)) * PAGE_TOKENS + (id % (TALK_KEYS / 8)) * 8 : 0));
    }
  };
  auto stash = [&](int which, int n0) {  // keys into their one place, values into place `which`
#pragma unroll
    for (int n = 0; n < KP; ++n) {
      const unsigned at = k_at[HALVES && n0 ? n + KCH - KP : n];
      if (at != TALK_NOWHERE) *reinterpret_cast<bf16x8*>(ks + (at >> 16) * 8) = kbuf[n];
    }
    if (n0) return;
#pragma unroll
    for (int n = 0; n < VCH; ++n) {
      const int id = threadIdx.x + n * TALK_PREFILL_THREADS;
      if (id < v_pieces) *reinterpret_cast<bf16x8*>(vs + which * L::V_ELEMS + (id / (TALK_KEYS / 8)) * VS + (id % (TALK_KEYS / 8)) * 8) = vbuf[n];
    }
  };
  f32x16 acc[DA];
#pragma unroll
  for (int dt = 0; dt < DA; ++dt)
#pragma unroll
    for (int v = 0; v < 16; ++v) acc[dt][v] = 0.f;
  float m = TALK_EMPTY, l = 0.f;
  const float scale2 = a.scale * TALK_LOG2E;
  const int key_row = 16 * (j >> 4) + 8 * ((j >> 2) & 1) + 4 * ((j >> 3) & 1) + (j & 3);
  const bf16* const kbase = ks + (size_t)key_row * KS + side * KH * 16 + half * 8;
  f32x4* const give = exchange + (size_t)wave * (OWN / 4) * WAVE + lane;
  const f32x4* const take = exchange + (size_t)(wave ^ 1) * (OWN / 4) * WAVE + lane;

  fetch(tile_first, 0);
  stash(0, 0);
  if (HALVES) {
    fetch(tile_first, KP);
    stash(0, KP);
  }
  fetch(tile_first < tile_last ? tile_first + 1 : tile_last, 0);
  block_sync_lds();
  for (int tile = tile_first; tile <= tile_last; ++tile) {
    const int cur = (tile - tile_first) & 1;
    const int key0 = tile * TALK_KEYS;
    const bool active = has_work && key0 <= wave_hi && key0 + TALK_KEYS - 1 >= wave_lo;  // uniform over the unit
    float own[OWN];  // scores of the tile's keys 8 half .. + 7 of 0 .. 15, of 16 .. 31, or both
    if (active) {
      f32x16 sc;
#pragma unroll
      for (int v = 0; v < 16; ++v) sc[v] = 0.f;
#pragma unroll
      for (int c = 0; c < KH; ++c) sc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(talk_load8(kbase + c * 16), qreg[c], sc, 0, 0, 0);
      if (SPLIT_VALUES) {
#pragma unroll
        for (int q = 0; q < OWN / 4; ++q) give[q * WAVE] = f32x4{sc[4 * q], sc[4 * q + 1], sc[4 * q + 2], sc[4 * q + 3]};
#pragma unroll
        for (int v = 0; v < OWN; ++v) own[v] = sc[v];
      } else if (side == 0) {  // uniform over the wave
        give[0] = f32x4{sc[8], sc[9], sc[10], sc[11]}, give[WAVE] = f32x4{sc[12], sc[13], sc[14], sc[15]};
#pragma unroll
        for (int v = 0; v < 8; ++v) own[v] = sc[v];
      } else {
        give[0] = f32x4{sc[0], sc[1], sc[2], sc[3]}, give[WAVE] = f32x4{sc[4], sc[5], sc[6], sc[7]};
#pragma unroll
        for (int v = 0; v < 8; ++v) own[v] = sc[8 + v];
      }
    }
    block_sync_lds();  // the handed-over sums are there; nobody reads this tile's keys any more
    if (tile < tile_last) stash(cur ^ 1, 0);
    // (past the end the last tile again: cheaper than a branch around loads)
    if (HALVES) fetch(tile < tile_last ? tile + 1 : tile_last, KP);
    else fetch(tile + 2 <= tile_last ? tile + 2 : tile_last, 0);
    if (active) {
      const int first = key0 + (SPLIT_VALUES ? 0 : 16 * side);
#pragma unroll
      for (int q = 0; q < OWN / 4; ++q) {
        const f32x4 o = take[q * WAVE];
#pragma unroll
        for (int e = 0; e < 4; ++e) own[4 * q + e] += o[e];
      }
      if (!(first + 2 * OWN - 1 <= full_hi && first >= full_lo)) {
#pragma unroll
        for (int v = 0; v < OWN; ++v) {
          const int key = first + 16 * (v >> 3) + 8 * half + (v & 7);
          own[v] = (key <= qpos && key >= qlo) ? own[v] : -INFINITY;
        }
      }
      float mx = own[0];
#pragma unroll
      for (int v = 1; v + 1 < OWN; v += 2) mx = talk_max3(mx, own[v], own[v + 1]);
      mx = talk_max2(mx, own[OWN - 1]);
      {
        const unsigned u = __float_as_uint(mx);
        const auto halves = __builtin_amdgcn_permlane32_swap(u, u, false, false);  // the column's other lane
        mx = talk_max2(__uint_as_float(halves[0]), __uint_as_float(halves[1]));
      }
      const float m_new = talk_max2(m, mx * scale2);
      const float alpha = __builtin_amdgcn_exp2f(m - m_new);
      m = m_new;
      float psum = 0.f;
#pragma unroll
      for (int v = 0; v < OWN; ++v) {
        own[v] = __builtin_amdgcn_exp2f(fmaf(own[v], scale2, -m_new));
        psum += own[v];
      }
      l = l * alpha + psum;
      if (__any(alpha != 1.f)) {  // the running maximum seldom moves after the first keys
#pragma unroll
        for (int dt = 0; dt < DA; ++dt) acc[dt] *= alpha;
      }
#pragma unroll
      for (int e = 0; e < OWN / 8; ++e) {
        const bf16x8 pmat = {(bf16)own[8 * e], (bf16)own[8 * e + 1], (bf16)own[8 * e + 2], (bf16)own[8 * e + 3],
                             (bf16)own[8 * e + 4], (bf16)own[8 * e + 5], (bf16)own[8 * e + 6], (bf16)own[8 * e + 7]};
        const bf16* vbase = vs + cur * L::V_ELEMS + (size_t)((SPLIT_VALUES ? side * DA * 32 : 0) + j) * VS + (SPLIT_VALUES ? 16 * e : 16 * side) + 8 * half;
#pragma unroll
        for (int dt = 0; dt < DA; ++dt)
          if (!SPLIT_VALUES || side * DA + dt < DT)  // uniform over the wave
            acc[dt] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(talk_load8(vbase + dt * 32 * VS), pmat, acc[dt], 0, 0, 0);
      }
    }
    if (HALVES) {
      if (tile < tile_last) stash(cur ^ 1, KP);
      fetch(tile + 2 <= tile_last ? tile + 2 : tile_last, 0);
    }
    block_sync_lds();  // the next tile's keys are there; this tile's values and the handed-over sums are read
  }
  // ---- the two waves of a unit meet: the second hands its result over, one run of 32 value channels after the other ----
  __syncthreads();  // the loads still under way, before the memory changes its use
  l += __shfl_xor(l, 32, WAVE);
  if constexpr (SPLIT_VALUES) {  // both waves have the whole sums, and channels of their own
    if (!valid) return;
    if (a.sink != nullptr) l += __builtin_amdgcn_exp2f(a.sink[h] * TALK_LOG2E - m);
    const float inv = l > 0.f ? 1.f / l : 0.f;
    bf16* orow = a.out + (size_t)t * a.out_stride + (size_t)h * a.vdim;
#pragma unroll
    for (int dt = 0; dt < DA; ++dt) {
#pragma unroll
      for (int q = 0; q < 4; ++q) {
        const int d = (side * DA + dt) * 32 + 8 * q + 4 * half;
        if (d < a.vdim)
          *reinterpret_cast<bf16x4*>(orow + d) = bf16x4{(bf16)(acc[dt][4 * q] * inv), (bf16)(acc[dt][4 * q + 1] * inv),
                                                        (bf16)(acc[dt][4 * q + 2] * inv), (bf16)(acc[dt][4 * q + 3] * inv)};
      }
    }
    return;
  }
  f32x4* const hand = reinterpret_cast<f32x4*>(talk_lds) + (size_t)unit * 5 * WAVE + lane;  // [unit][4 + 1][lane]
  float f0 = 0.f, f1 = 0.f;  // what the two results are multiplied by
#pragma unroll
  for (int dt = 0; dt < DA; ++dt) {
    if (side == 1) {
#pragma unroll
      for (int q = 0; q < 4; ++q) hand[q * WAVE] = f32x4{acc[dt][4 * q], acc[dt][4 * q + 1], acc[dt][4 * q + 2], acc[dt][4 * q + 3]};
      if (dt == 0) hand[4 * WAVE] = f32x4{m, l, 0.f, 0.f};
    }
    __syncthreads();
    if (side == 0 && valid) {
      if (dt == 0) {
        const f32x4 other = hand[4 * WAVE];
        float top = fmaxf(m, other[0]);
        if (a.sink != nullptr) top = fmaxf(top, a.sink[h] * TALK_LOG2E);
        f0 = __builtin_amdgcn_exp2f(m - top), f1 = __builtin_amdgcn_exp2f(other[0] - top);
        float sum = l * f0 + other[1] * f1;
        if (a.sink != nullptr) sum += __builtin_amdgcn_exp2f(a.sink[h] * TALK_LOG2E - top);
        const float inv = sum > 0.f ? 1.f / sum : 0.f;
        f0 *= inv, f1 *= inv;
      }
      bf16* orow = a.out + (size_t)t * a.out_stride + (size_t)h * a.vdim;
#pragma unroll
      for (int q = 0; q < 4; ++q) {
        const int d = dt * 32 + 8 * q + 4 * half;
        const f32x4 o = hand[q * WAVE];
        if (d < a.vdim)
          *reinterpret_cast<bf16x4*>(orow + d) =
              bf16x4{(bf16)(acc[dt][4 * q] * f0 + o[0] * f1), (bf16)(acc[dt][4 * q + 1] * f0 + o[1] * f1),
                     (bf16)(acc[dt][4 * q + 2] * f0 + o[2] * f1), (bf16)(acc[dt][4 * q + 3] * f0 + o[3] * f1)};
      }
    }
    __syncthreads();  // the memory carries the next run
  }
}

// Decode steps: a block per (token, 16 heads, split).  The visible keys of the token's sequence are cut into tiles of 32,
// dealt over the splits' waves in turn; a wave's columns are the 16 heads.  All columns run against every kv head's values,
// with the probabilities of the other kv heads' columns set to zero, so the sums meet in one set of accumulators.  The
// waves of a block merge in LDS; with several splits the block leaves (maximum, sum, unnormalised result) in the workspace
// and talking_merge_kernel joins them.
#define TALK_DECODE_WAVES 4

template <int KC2, int DT2>
__global__ void __launch_bounds__(TALK_DECODE_WAVES* WAVE)
    talking_decode_kernel(TalkArgs a, int n_splits, float* __restrict__ workspace) {
  constexpr int KW = KC2 * 32, KS = KW + TALK_PAD;
  constexpr int THREADS = TALK_DECODE_WAVES * WAVE;
  constexpr int QBYTES = 16 * KS * 2, OS = DT2 * 16 + 4, OBYTES = TALK_DECODE_WAVES * 16 * OS * 4;
  __shared__ __attribute__((aligned(16))) unsigned char lds[QBYTES > OBYTES ? QBYTES : OBYTES];
  __shared__ float wm[TALK_DECODE_WAVES][16], wl[TALK_DECODE_WAVES][16];
  const int t = blockIdx.x, split = blockIdx.y, h0 = blockIdx.z * 16;
  const int seq = uniform_load(a.seq_of_token + t);
  const int wave = threadIdx.x / WAVE, lane = threadIdx.x & (WAVE - 1);
  const int r = lane & 15, g = lane >> 4;
  const int row = a.kvheads * a.dim, per = a.nheads / a.kvheads;
  float* const part = workspace + ((size_t)t * n_splits + split) * a.nheads * (a.vdim + 2);  // [heads][vdim], then [heads][2]
  if (seq < 0) {
    // a padding row: zeros; the merge kernel skips it as well
    if (n_splits == 1)
      for (int i = threadIdx.x; i < 16 * a.vdim; i += THREADS)
        if (h0 + i / a.vdim < a.nheads) a.out[(size_t)t * a.out_stride + (size_t)h0 * a.vdim + i] = (bf16)0.f;
    return;
  }
  // the mixed queries of the block's heads, in LDS for all waves
  bf16* const qs = reinterpret_cast<bf16*>(lds);
  for (int i = threadIdx.x; i < 16 * (KW / 8); i += THREADS) {
    const int hh = i / (KW / 8), k = (i % (KW / 8)) * 8;
    bf16x8 v = {0, 0, 0, 0, 0, 0, 0, 0};
    if (h0 + hh < a.nheads && k < row) {
      const int c = k / a.dim;
      v = talk_mixed_query(a.q + (size_t)t * a.q_stride, a.talk + (size_t)(h0 + hh) * a.nheads, c, k - c * a.dim, per, a.dim);
    }
    *reinterpret_cast<bf16x8*>(qs + hh * KS + k) = v;
  }
  __syncthreads();
  bf16x8 qreg[KC2];
#pragma unroll
  for (int c = 0; c < KC2; ++c) qreg[c] = talk_load8(qs + r * KS + c * 32 + g * 8);

  const int pos = uniform_load(a.positions + t);
  const int lo = talk_first_key(pos, a.window);
  const int* bt = a.block_table + (size_t)seq * a.table_stride;
  const size_t page_elems = (size_t)a.kvheads * PAGE_TOKENS * a.dim, vpage_elems = (size_t)a.kvheads * PAGE_TOKENS * a.vdim;
  const int tile_first = lo / TALK_KEYS, tile_last = pos / TALK_KEYS;
  const float scale2 = a.scale * TALK_LOG2E;
  const int key_a = (r >> 2) * 8 + (r & 3);
  const int my_kv = (h0 + r) / per;  // this lane's column reads the values of this kv head

  f32x4 acc[DT2];
#pragma unroll
  for (int dt = 0; dt < DT2; ++dt) acc[dt] = f32x4{0.f, 0.f, 0.f, 0.f};
  float m = TALK_EMPTY, l = 0.f;
  for (int tile = tile_first + split * TALK_DECODE_WAVES + wave; tile <= tile_last; tile += n_splits * TALK_DECODE_WAVES) {
    const int key0 = tile * TALK_KEYS;
    const size_t phys = readable_page(uniform_load(bt + key0 / PAGE_TOKENS));
    const bf16* kp = a.k_cache + phys * page_elems + (size_t)(key0 % PAGE_TOKENS) * a.dim;
    const bf16* vp = a.v_cache + phys * vpage_elems + key0 % PAGE_TOKENS;
    f32x4 sa = f32x4{0.f, 0.f, 0.f, 0.f}, sb = f32x4{0.f, 0.f, 0.f, 0.f};
    constexpr int STEP = KC2 % 8 == 0 ? 8 : 4;  // k-steps whose keys are asked for together
    static_assert(KC2 % STEP == 0, "whole runs of k-steps");
#pragma unroll
    for (int c0 = 0; c0 < KC2; c0 += STEP) {
      bf16x8 ka[STEP], kb[STEP];
#pragma unroll
      for (int c = 0; c < STEP; ++c) {
        int k = (c0 + c) * 32 + g * 8;
        if (k >= row) k = 0;  // the query is zero there
        const int kv = k / a.dim;
        const bf16* src = kp + (size_t)kv * PAGE_TOKENS * a.dim + (k - kv * a.dim);
        ka[c] = talk_load8(src + (size_t)key_a * a.dim);
        kb[c] = talk_load8(src + (size_t)(key_a + 4) * a.dim);
      }
#pragma unroll
      for (int c = 0; c < STEP; ++c) {
        sa = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ka[c], qreg[c0 + c], sa, 0, 0, 0);
        sb = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kb[c], qreg[c0 + c], sb, 0, 0, 0);
      }
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int ja = key0 + g * 8 + i, jb = ja + 4;
      sa[i] = (ja <= pos && ja >= lo) ? sa[i] : -INFINITY;
      sb[i] = (jb <= pos && jb >= lo) ? sb[i] : -INFINITY;
    }
    float mx = talk_max3(talk_max3(sa[0], sa[1], sa[2]), talk_max3(sa[3], sb[0], sb[1]), talk_max2(sb[2], sb[3]));
    mx = fmaxf(mx, __shfl_xor(mx, 16, WAVE));
    mx = fmaxf(mx, __shfl_xor(mx, 32, WAVE));
    const float m_new = talk_max2(m, mx * scale2);
    const float alpha = __builtin_amdgcn_exp2f(m - m_new);
    m = m_new;
    float pa[4], pb[4], psum = 0.f;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      pa[i] = __builtin_amdgcn_exp2f(fmaf(sa[i], scale2, -m_new));
      pb[i] = __builtin_amdgcn_exp2f(fmaf(sb[i], scale2, -m_new));
      psum += pa[i] + pb[i];
    }
    l = l * alpha + psum;
    const bf16x8 pmat = {(bf16)pa[0], (bf16)pa[1], (bf16)pa[2], (bf16)pa[3], (bf16)pb[0], (bf16)pb[1], (bf16)pb[2], (bf16)pb[3]};
    const bf16x8 none = {0, 0, 0, 0, 0, 0, 0, 0};
    if (__any(alpha != 1.f)) {
#pragma unroll
      for (int dt = 0; dt < DT2; ++dt) acc[dt] *= alpha;
    }
    for (int c = h0 / per; c < a.kvheads && c * per < h0 + 16; ++c) {  // the kv heads of the block's heads
      const bf16x8 pc = my_kv == c ? pmat : none;
      bf16x8 v[DT2];
#pragma unroll
      for (int dt = 0; dt < DT2; ++dt) {
        const int d = dt * 16 + r;
        v[dt] = talk_load8(vp + ((size_t)c * a.vdim + (d < a.vdim ? d : 0)) * PAGE_TOKENS + g * 8);
      }
#pragma unroll
      for (int dt = 0; dt < DT2; ++dt) acc[dt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(v[dt], pc, acc[dt], 0, 0, 0);
    }
  }
  l += __shfl_xor(l, 16, WAVE);
  l += __shfl_xor(l, 32, WAVE);
  __syncthreads();  // every wave holds its queries: the memory changes its use
  float* const os = reinterpret_cast<float*>(lds);  // [wave][head][OS]
#pragma unroll
  for (int dt = 0; dt < DT2; ++dt) *reinterpret_cast<f32x4*>(os + (size_t)(wave * 16 + r) * OS + dt * 16 + g * 4) = acc[dt];
  if (g == 0) wm[wave][r] = m, wl[wave][r] = l;
  __syncthreads();
  for (int i = threadIdx.x; i < 16 * a.vdim; i += THREADS) {
    const int hh = i / a.vdim, d = i % a.vdim;
    if (h0 + hh >= a.nheads) break;  // heads ascend with i
    float top = wm[0][hh];
#pragma unroll
    for (int w = 1; w < TALK_DECODE_WAVES; ++w) top = fmaxf(top, wm[w][hh]);
    float sum = 0.f, o = 0.f;
#pragma unroll
    for (int w = 0; w < TALK_DECODE_WAVES; ++w) {
      const float f = __builtin_amdgcn_exp2f(wm[w][hh] - top);
      sum = fmaf(wl[w][hh], f, sum);
      o = fmaf(os[(size_t)(w * 16 + hh) * OS + d], f, o);
    }
    if (n_splits == 1) {
      if (a.sink != nullptr) {
        const float s2 = a.sink[h0 + hh] * TALK_LOG2E;
        sum += __builtin_amdgcn_exp2f(s2 - top);
      }
      a.out[(size_t)t * a.out_stride + (size_t)(h0 + hh) * a.vdim + d] = (bf16)(sum > 0.f ? o / sum : 0.f);
    } else {
      part[(size_t)(h0 + hh) * a.vdim + d] = o;
      if (d == 0) {
        float* ml = part + (size_t)a.nheads * a.vdim + 2 * (h0 + hh);
        ml[0] = top, ml[1] = sum;
      }
    }
  }
}

// joins the splits of a (token, head): a thread per output element
__global__ void __launch_bounds__(256) talking_merge_kernel(TalkArgs a, int n_splits, const float* __restrict__ workspace) {
  const int t = blockIdx.x;
  const int i = blockIdx.y * 256 + threadIdx.x;
  if (i >= a.nheads * a.vdim) return;
  bf16* o = a.out + (size_t)t * a.out_stride + i;
  if (a.seq_of_token[t] < 0) {
    *o = (bf16)0.f;
    return;
  }
  const int h = i / a.vdim;
  const size_t size = (size_t)a.nheads * (a.vdim + 2);
  const float* part = workspace + (size_t)t * n_splits * size;
  const float* ml = part + (size_t)a.nheads * a.vdim + 2 * h;
  float top = a.sink != nullptr ? a.sink[h] * TALK_LOG2E : TALK_EMPTY;
  for (int s = 0; s < n_splits; ++s) top = fmaxf(top, ml[(size_t)s * size]);
  float sum = a.sink != nullptr ? __builtin_amdgcn_exp2f(a.sink[h] * TALK_LOG2E - top) : 0.f, acc = 0.f;
  for (int s = 0; s < n_splits; ++s) {
    const float f = __builtin_amdgcn_exp2f(ml[(size_t)s * size] - top);
    sum = fmaf(ml[(size_t)s * size + 1], f, sum);
    acc = fmaf(part[(size_t)s * size + i], f, acc);
  }
  *o = (bf16)(sum > 0.f ? acc / sum : 0.f);
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

// ---- the matrix-core kernels -----------------------------------------------------------------------------------------------
static int talking_padded_row(int kvheads, int dim) {
  const int row = kvheads * dim;
  const int sizes[] = {128, 256, 384, 512, 1024};
  for (int s : sizes)
    if (row <= s) return s;
  return 0;
}

extern "C" int fmsamd_talking_attn_mfma_fits(int kvheads, int head_dim, int value_dim) {
  return head_dim % 8 == 0 && value_dim % 8 == 0 && value_dim <= 128 && talking_padded_row(kvheads, head_dim) > 0;
}

// heads of a kv head that share a prompt block: the largest of 4, 2, 1 that divides them
static int talking_heads_of_block(int nheads, int kvheads) {
  const int per = nheads / kvheads;
  return per % 4 == 0 ? 4 : (per % 2 == 0 ? 2 : 1);
}

extern "C" int fmsamd_talking_attn_qblock(int nheads, int kvheads) { return 32 * TALK_UNITS / talking_heads_of_block(nheads, kvheads); }

static int talking_mfma_common(const char* name, const TalkArgs& a) {
  if (talking_common(name, a.n_tokens, a.nheads, a.kvheads, a.dim, a.vdim, a.q_stride, a.out_stride, a.talk)) return -1;
  FMS_REQUIRE(fmsamd_talking_attn_mfma_fits(a.kvheads, a.dim, a.vdim), "%s: %d kv heads of %d with values of %d do not fit the matrix-core kernels",
              name, a.kvheads, a.dim, a.vdim);
  FMS_REQUIRE(a.q_stride % 8 == 0 && (uintptr_t)a.q % 16 == 0 && (uintptr_t)a.k_cache % 16 == 0 && (uintptr_t)a.v_cache % 16 == 0 &&
                  a.out_stride % 4 == 0 && (uintptr_t)a.out % 8 == 0,
              "%s: rows and caches must start at multiples of 16 bytes", name);
  FMS_REQUIRE(a.scale > 0.f, "%s: the scale %g must be positive", name, (double)a.scale);
  return 0;
}

#define FMS_TALK_SIZES(KW, DT, CALL)       \
  do {                                     \
    switch (KW) {                          \
      case 128: FMS_TALK_VALUES(8, DT, CALL); break;  \
      case 256: FMS_TALK_VALUES(16, DT, CALL); break; \
      case 384: FMS_TALK_VALUES(24, DT, CALL); break; \
      case 512: FMS_TALK_VALUES(32, DT, CALL); break; \
      default: FMS_TALK_VALUES(64, DT, CALL); break;  \
    }                                      \
  } while (0)
#define FMS_TALK_VALUES(KC, DT, CALL)  \
  do {                                 \
    if (DT == 1) CALL(KC, 1);          \
    else if (DT == 2) CALL(KC, 2);     \
    else if (DT == 3) CALL(KC, 3);     \
    else CALL(KC, 4);                  \
  } while (0)

extern "C" int fmsamd_talking_attn_prefill(const void* q, long q_stride, void* out, long out_stride, const int* positions,
                                           const int* seq_of_token, const int* qblock_start, const int* qblock_len, int n_qblocks,
                                           int qblock_tokens, const int* block_table, int table_stride, const void* k_cache,
                                           const void* v_cache, const float* talk, const float* sink, int n_tokens, int nheads,
                                           int kvheads, int head_dim, int value_dim, float scale, int window, hipStream_t stream) {
  if (n_tokens == 0 || n_qblocks == 0) return 0;
  TalkArgs a{(const bf16*)q, q_stride, (bf16*)out, out_stride, positions, seq_of_token, block_table, table_stride, (const bf16*)k_cache,
             (const bf16*)v_cache, talk, sink, n_tokens, nheads, kvheads, head_dim, value_dim, scale, window};
  if (talking_mfma_common("talking_attn_prefill", a)) return -1;
  FMS_REQUIRE(qblock_tokens == fmsamd_talking_attn_qblock(nheads, kvheads), "talking_attn_prefill: query blocks of %d tokens, the kernel takes %d",
              qblock_tokens, fmsamd_talking_attn_qblock(nheads, kvheads));
  const int hb = talking_heads_of_block(nheads, kvheads);
  const long blocks = (long)n_qblocks * kvheads * (nheads / kvheads / hb);
  FMS_REQUIRE(blocks < (1L << 31), "talking_attn_prefill: too many blocks");
  FMS_REQUIRE((long)hb * nheads * 4 <= TALK_UNITS * 2 * WAVE * 8 * 4, "talking_attn_prefill: %d heads", nheads);
  const int kw = talking_padded_row(kvheads, head_dim), dt = ceil_div(value_dim, 32);
#define FMS_TP(KC, DT)                                                                                                                \
  do {                                                                                                                                \
    constexpr int bytes = TalkPrefillLds<KC, DT>::BYTES;                                                                              \
    static const hipError_t sized = hipFuncSetAttribute(reinterpret_cast<const void*>(talking_prefill_kernel<KC, DT>),                \
                                                        hipFuncAttributeMaxDynamicSharedMemorySize, bytes);                           \
    FMS_REQUIRE(sized == hipSuccess, "talking_attn_prefill: %d bytes of LDS refused: %s", bytes, hipGetErrorString(sized));           \
    talking_prefill_kernel<KC, DT><<<(unsigned)blocks, TALK_PREFILL_THREADS, bytes, stream>>>(a, qblock_start, qblock_len, n_qblocks, hb); \
  } while (0)
  FMS_TALK_SIZES(kw, dt, FMS_TP);
#undef FMS_TP
  FMS_LAUNCH_CHECK("talking_attn_prefill");
  return 0;
}

extern "C" long fmsamd_talking_attn_workspace(int n_tokens, int nheads, int value_dim, int n_splits) {
  return n_splits > 1 ? (long)n_tokens * n_splits * nheads * (value_dim + 2) * 4 : 0;
}

extern "C" int fmsamd_talking_attn_decode(const void* q, long q_stride, void* out, long out_stride, void* workspace, long workspace_bytes,
                                          const int* positions, const int* seq_of_token, const int* block_table, int table_stride,
                                          const void* k_cache, const void* v_cache, const float* talk, const float* sink, int n_tokens,
                                          int nheads, int kvheads, int head_dim, int value_dim, float scale, int window, int n_splits,
                                          hipStream_t stream) {
  if (n_tokens == 0) return 0;
  TalkArgs a{(const bf16*)q, q_stride, (bf16*)out, out_stride, positions, seq_of_token, block_table, table_stride, (const bf16*)k_cache,
             (const bf16*)v_cache, talk, sink, n_tokens, nheads, kvheads, head_dim, value_dim, scale, window};
  if (talking_mfma_common("talking_attn_decode", a)) return -1;
  FMS_REQUIRE(n_splits >= 1 && n_splits <= 65535 && ceil_div(nheads, 16) <= 65535, "talking_attn_decode: %d splits of %d heads", n_splits, nheads);
  FMS_REQUIRE(workspace_bytes >= fmsamd_talking_attn_workspace(n_tokens, nheads, value_dim, n_splits) && (n_splits == 1 || workspace != nullptr),
              "talking_attn_decode: the workspace is too small");
  const dim3 grid(n_tokens, n_splits, ceil_div(nheads, 16));
  const int kw = talking_padded_row(kvheads, head_dim), dt = ceil_div(value_dim, 32);
#define FMS_TD(KC, DT) talking_decode_kernel<KC / 2, DT * 2><<<grid, TALK_DECODE_WAVES * WAVE, 0, stream>>>(a, n_splits, (float*)workspace)
  FMS_TALK_SIZES(kw, dt, FMS_TD);
#undef FMS_TD
  FMS_LAUNCH_CHECK("talking_attn_decode");
  if (n_splits > 1) {
    FMS_REQUIRE(ceil_div((long)nheads * value_dim, 256) <= 65535, "talking_attn_decode: too many output elements");
    talking_merge_kernel<<<dim3(n_tokens, ceil_div((long)nheads * value_dim, 256)), 256, 0, stream>>>(a, n_splits, (const float*)workspace);
    FMS_LAUNCH_CHECK("talking_merge");
  }
  return 0;
}
