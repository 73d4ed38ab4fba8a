// The state-space recurrence of Mamba-2: per head a matrix S [value channels P, state rows N],
//
//   S <- exp(-exp(a_log) d) S + d x B^T,   y = S C + skip x,   d = softplus(dt + dt_bias)
//
// with x of P channels per head, B and C of N channels per group of heads; everything in float32.
//
//   ssd_scan:         token by token (decode steps, short portions).  The rows of S never mix, so 16 lanes share a value
//                     channel, each with a run of its N entries in registers.
//   gated_group_norm: y * silu(z), each of `parts` equal parts of the row over its own root mean square, times a weight.
//
// The state is kept [slot][head][value channel][state row], so that a lane's entries are contiguous.
#include "common.h"
#include "fmsamd.h"

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

// A block per (token, part); the part's gated values wait in registers (up to 16 a thread, the rest is formed again).
template <typename T, typename W>
__global__ void __launch_bounds__(1024)
    gated_group_norm_kernel(const float* __restrict__ y, const float* __restrict__ z, long ldz, const W* __restrict__ weight, float eps,
                            T* __restrict__ out, const int* __restrict__ seq_of_token, int cols, int size) {
  __shared__ float scratch[17];
  constexpr int KEEP = 16;
  const int t = blockIdx.x, c0 = blockIdx.y * size;
  if (seq_of_token[t] < 0) return;
  const float* yr = y + (size_t)t * cols + c0;
  const float* zr = z + (size_t)t * ldz + c0;
  const W* wr = weight + c0;
  T* o = out + (size_t)t * cols + c0;
  auto gated = [&](int i) {
    const float g = zr[i];
    return yr[i] * (g / (1.f + expf(-g)));
  };
  float keep[KEEP], s = 0.f;
#pragma unroll
  for (int n = 0; n < KEEP; ++n) {
    const int i = threadIdx.x + n * blockDim.x;
    keep[n] = i < size ? gated(i) : 0.f;
    s = fmaf(keep[n], keep[n], s);
  }
  for (int i = threadIdx.x + KEEP * blockDim.x; i < size; i += blockDim.x) {
    const float v = gated(i);
    s = fmaf(v, v, s);
  }
  const float inv = 1.f / sqrtf(block_sum(s, scratch) / (float)size + eps);
#pragma unroll
  for (int n = 0; n < KEEP; ++n) {
    const int i = threadIdx.x + n * blockDim.x;
    if (i < size) o[i] = from_f32<T>(keep[n] * inv * to_f32(wr[i]));
  }
  for (int i = threadIdx.x + KEEP * blockDim.x; i < size; i += blockDim.x) o[i] = from_f32<T>(gated(i) * inv * to_f32(wr[i]));
}

extern "C" int fmsamd_gated_group_norm(const float* y, const float* z, long ldz, const void* weight, int weight_dtype, int parts, float eps,
                                       void* out, int out_dtype, const int* seq_of_token, int n_tokens, int cols, hipStream_t stream) {
  if (n_tokens == 0) return 0;
  FMS_REQUIRE(n_tokens > 0 && cols > 0 && parts > 0 && cols % parts == 0 && ldz >= cols, "gated_group_norm: %d parts of %d channels", parts, cols);
  FMS_REQUIRE(parts <= 65535, "gated_group_norm: %d parts are too many for one launch", parts);
  const int size = cols / parts;
  const int threads = size >= 2048 ? 512 : (size >= 512 ? 256 : 64);
  const dim3 grid(n_tokens, parts);
#define FMS_GGN(T, W)                                                                                                             \
  gated_group_norm_kernel<T, W><<<grid, threads, 0, stream>>>(y, z, ldz, (const W*)weight, eps, (T*)out, seq_of_token, cols, size)
  if (out_dtype == FMS_F32 && weight_dtype == FMS_F32) FMS_GGN(float, float);
  else if (out_dtype == FMS_BF16 && weight_dtype == FMS_F32) FMS_GGN(bf16, float);
  else if (out_dtype == FMS_BF16 && weight_dtype == FMS_BF16) FMS_GGN(bf16, bf16);
  else if (out_dtype == FMS_F32 && weight_dtype == FMS_BF16) FMS_GGN(float, bf16);
  else FMS_REQUIRE(false, "gated_group_norm: unknown dtypes %d, %d", out_dtype, weight_dtype);
#undef FMS_GGN
  FMS_LAUNCH_CHECK("gated_group_norm");
  return 0;
}
