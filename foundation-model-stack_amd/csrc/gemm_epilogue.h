// What the bfloat16 products for few rows (gemm.hip: at most 16 rows; gemm_wide.hip: 17 to 192) do with a
// finished output element, and the arguments of those epilogues.
#pragma once

#include "common.h"
#include "fmsamd.h"

__device__ __forceinline__ float sk_activate(float x, int kind) {
  if (kind == FMS_ACT_SILU) return x / (1.f + __expf(-x));  // the one every served model has: the fast exponential
  return fms_activate(x, kind);
}

// The activations that a plain product finishes with (the others are a kernel of their own behind it: a switch over all of
// them at every store would cost every product).
__device__ __forceinline__ float sk_plain(float x, int act) {
  if (act == FMS_ACT_IDENTITY) return x;
  const float r = fmaxf(x, 0.f);
  return act == FMS_ACT_RELU2 ? r * r : r;
}

// What a product finishes an element with: an activation, and for the clamped gated unit (FMS_ACT_CLAMPED_GATE, gated
// products only) its constants.
struct OutAct {
  int kind;
  float limit, alpha, shift;
};
static inline OutAct plain_act(int kind) { return OutAct{kind, 0.f, 0.f, 0.f}; }

// The gated unit: act(gate) * up, or g sigmoid(alpha g) (u + shift) with g = min(gate, limit), u = clamp(up, -limit, limit).
__device__ __forceinline__ float sk_gated(float gate, float up, const OutAct& a) {
  if (a.kind == FMS_ACT_CLAMPED_GATE) return clamped_gate(gate, up, a.limit, a.alpha, a.shift);
  return sk_activate(gate, a.kind) * up;
}

// What the skinny kernel does with a finished output element.
#define EPI_PLAIN 0  // store act(product + bias), act one of identity, relu and its square
#define EPI_GATED 1  // the block's second tile is the "up" half: out = act(first) * second (or the clamped unit), N is the hidden size
#define EPI_ROPE 2   // the output row is [queries | keys | values] of attention: rotate q and k, store q, and
                     // write k and v into their cache pages (layout: see rope.hip)
#define EPI_RESID 3  // add the product to the float32 residual stream in place, store the new stream times the
                     // next norm's weight in the activation type, and leave the rows' sums of squares by tile

// The rows of x are not yet divided by their root mean square: the kernel that made them left, for each
// row, `count` partial sums of squares (partials[m * count + i]).  The product is multiplied by
// rsqrt(sum / width + eps) of its row before the bias.  partials == null: the rows are taken as they are.
struct RowScale {
  const float* partials;
  int count;
  float inv_width, eps;
};

struct ResidEpilogue {
  float* resid;  // [M, N] float32, read and written
  long ldr;
  const void* norm_w;  // [N] or null
  int norm_w_f32;
  float* partials;  // [M, tiles]: sum over the tile's 16 columns of the new stream squared
  int tiles;
};

struct RopeEpilogue {
  const int* positions;     // [M]
  const int* seq_of_token;  // [M], -1: padding row
  const int* block_table;
  int table_stride;
  const float* cos_t;  // [max_pos, rot_dim/2] or null
  const float* sin_t;
  int rot_dim, max_pos;
  bf16* k_cache;  // null: queries only
  bf16* v_cache;
  int nheads, kvheads, head_dim;
};


#define FMS_SKINNY_MAX_ROWS 192

// ---- 17 to 192 rows (gemm_wide.hip) ------------------------------------------
// The product runs as two kernels: blocks of 128 weight rows times a slice of K leave float32 partial sums
// in a workspace [slices][M][rows]; a second kernel adds the slices in a fixed order and applies the epilogue.
// `rows` counts all rows of W (for the gated product both halves).
long wide_workspace_bytes(int M, int rows, int K);
int wide_product(int epi, const void* x, long ldx, const void* w, const void* bias, int bias_dtype, void* out,
                 int out_dtype, long ldo, int M, int N, int K, int tile2_offset, OutAct act, RowScale scale,
                 RopeEpilogue rope, ResidEpilogue res, void* workspace, long workspace_bytes, hipStream_t stream);
