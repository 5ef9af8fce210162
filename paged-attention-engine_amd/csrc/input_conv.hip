// What a sublayer reads when a short convolution over time stands in front of it:
//
//   rows[t] = T(x_t + sum_b w[taps - 1 - b] * x_(t - b))      per channel, b = 0 .. taps - 1, zeros before the sequence
//
// with x the float32 residual stream.  A request's state holds its last keep = taps - 1 inputs as a ring: the input at
// position p lies at ring[p % keep] (float32, [keep][hidden] per slot), so a token writes one row and moves none.
//
//   input_conv           rows of a step's runs of tokens, tile by tile; the ring is read and moved on in the same kernel
//   norm_join_conv       for steps in which every sequence brings one token: a sublayer's output joins the stream through
//                        its norm, x <- x + scale * y / sqrt(mean(y^2) + eps) * g, and the rows of the convolution in
//                        front of the next sublayer are formed on the way (one workgroup a row)
//
// Filters are float32 [taps][hidden].  Sums are float32; a value is rounded once, when `rows` is written.
#include "common.h"
#include "api.h"

template <typename T, int W>
__device__ __forceinline__ void conv_store(T* p, const float (&v)[4]) {
  if (W == 1) {
    p[0] = from_f32<T>(v[0]);
  } else if (sizeof(T) == 4) {
    *reinterpret_cast<float4*>((float*)p) = make_float4(v[0], v[1], v[2], v[3]);
  } else {
    bf16_t h[4] = {__float2bfloat16(v[0]), __float2bfloat16(v[1]), __float2bfloat16(v[2]), __float2bfloat16(v[3])};
    *reinterpret_cast<uint2*>((bf16_t*)p) = *reinterpret_cast<const uint2*>(h);
  }
}

template <int W>
__device__ __forceinline__ void conv_load(const float* p, float (&v)[4]) {
  if (W == 1) {
    v[0] = p[0];
  } else {
    const float4 x = *reinterpret_cast<const float4*>(p);
    v[0] = x.x; v[1] = x.y; v[2] = x.z; v[3] = x.w;
  }
}

// tiles[i] = (table row of the sequence, first flat row, rows, rows of the sequence in this step before the tile);
// runs[s] = (first flat row, rows in this step, tokens held before, unused).  A thread has W channels of a tile.  A tile
// that is not its sequence's first begins at least `keep` rows into the step, so only first tiles look into the ring, and
// they alone write it, after they have read it.
// TAPS > 0: that many taps, the inputs in registers; 0: any number, inputs read again for every tap.
template <typename T, int W, int TAPS, int ROWS>
__global__ __launch_bounds__(128) void input_conv_kernel(T* __restrict__ rows, const float* __restrict__ x,
                                                         const float* __restrict__ filters, float* ring_base,
                                                         int64_t slot_stride, const int4* __restrict__ tiles,
                                                         const int4* __restrict__ runs, const int* __restrict__ slots,
                                                         int taps_any, int hidden) {
  const int c = (blockIdx.y * 128 + threadIdx.x) * W;
  if (c >= hidden) return;
  const int4 tile = tiles[blockIdx.x];
  const int4 run = runs[tile.x];
  const int taps = TAPS > 0 ? TAPS : taps_any, keep = taps - 1;
  float* ring = ring_base + (int64_t)slots[tile.x] * slot_stride + c;
  const int pos0 = run.z + tile.w;  // position of the tile's first row
  const float* src = x + (int64_t)tile.y * hidden + c;
  T* dst = rows + (int64_t)tile.y * hidden + c;
  // the input `back` rows before row r of the tile
  auto input = [&](int r, int back, float (&v)[4]) {
    const int at = r - back;
    if (at + tile.w >= 0) {
      conv_load<W>(src + (int64_t)at * hidden, v);
    } else if (pos0 + at >= 0) {
      conv_load<W>(ring + (int64_t)((pos0 + at) % keep) * hidden, v);
    } else {
#pragma unroll
      for (int e = 0; e < W; ++e) v[e] = 0.f;
    }
  };
  if (TAPS > 0) {
    constexpr int KEEP = TAPS > 0 ? TAPS - 1 : 0;
    float in[KEEP + ROWS][4], w[KEEP + 1][4];
#pragma unroll
    for (int b = 0; b < KEEP; ++b) input(0, KEEP - b, in[b]);
#pragma unroll
    for (int r = 0; r < ROWS; ++r)
      if (r < tile.z) conv_load<W>(src + (int64_t)r * hidden, in[KEEP + r]);
#pragma unroll
    for (int j = 0; j < TAPS; ++j) conv_load<W>(filters + (int64_t)j * hidden + c, w[j]);
#pragma unroll
    for (int r = 0; r < ROWS; ++r) {
      if (r >= tile.z) break;
      float v[4];
#pragma unroll
      for (int e = 0; e < W; ++e) {
        float sum = 0.f;
#pragma unroll
        for (int j = 0; j < TAPS; ++j) sum = fmaf(w[j][e], in[r + j][e], sum);
        v[e] = in[KEEP + r][e] + sum;
      }
      conv_store<T, W>(dst + (int64_t)r * hidden, v);
    }
  } else {
    for (int r = 0; r < tile.z; ++r) {
      float sum[4] = {0.f, 0.f, 0.f, 0.f}, in[4] = {0.f, 0.f, 0.f, 0.f};
      for (int j = 0; j < taps; ++j) {
        float w[4];
        conv_load<W>(filters + (int64_t)j * hidden + c, w);
        input(r, keep - j, in);
#pragma unroll
        for (int e = 0; e < W; ++e) sum[e] = fmaf(w[e], in[e], sum[e]);
      }
#pragma unroll
      for (int e = 0; e < W; ++e) sum[e] += in[e];  // the last tap's input is the token's own
      conv_store<T, W>(dst + (int64_t)r * hidden, sum);
    }
  }
  if (tile.w == 0 && keep > 0) {
    const int n = run.y < keep ? run.y : keep;
    for (int i = run.y - n; i < run.y; ++i) {
      float v[4];
      conv_load<W>(src + (int64_t)i * hidden, v);
      float* to = ring + (int64_t)((run.z + i) % keep) * hidden;
#pragma unroll
      for (int e = 0; e < W; ++e) to[e] = v[e];
    }
  }
}

// Rows a tile for that many taps.
extern "C" int pae_input_conv_tile_rows(int taps) { return taps <= 8 ? 8 : taps - 1; }

extern "C" int pae_input_conv(int dtype, void* rows, const float* x, const float* filters, float* ring, int64_t slot_stride,
                              const int* tiles, int num_tiles, const int* runs, const int* slots, int taps, int hidden,
                              hipStream_t stream) {
  PAE_REQUIRE(taps >= 1 && taps <= 64, "input convolution: %d taps (1..64)", taps);
  PAE_REQUIRE(hidden > 0 && rows && x && filters && tiles && runs && slots, "input convolution: missing operands");
  PAE_REQUIRE(taps == 1 || (ring && slot_stride >= (int64_t)(taps - 1) * hidden), "input convolution: %d taps need the requests' state", taps);
  PAE_REQUIRE(dtype == PAE_F32 || dtype == PAE_BF16, "input convolution: unknown dtype code %d", dtype);
  if (num_tiles <= 0) return 0;
  const bool vec = hidden % 4 == 0 && (uintptr_t)x % 16 == 0 && (uintptr_t)rows % 16 == 0 && (uintptr_t)filters % 16 == 0 &&
                   (uintptr_t)ring % 16 == 0 && slot_stride % 4 == 0;
  const int width = vec ? 4 : 1;
  dim3 grid(num_tiles, (hidden + 128 * width - 1) / (128 * width));
#define CONV_AS(T, W, TAPS)                                                                                        \
  input_conv_kernel<T, W, TAPS, 8><<<grid, 128, 0, stream>>>((T*)rows, x, filters, ring, slot_stride,              \
                                                             (const int4*)tiles, (const int4*)runs, slots, taps, hidden)
#define CONV_BY_TAPS(T, W)                \
  switch (taps) {                         \
    case 2: CONV_AS(T, W, 2); break;      \
    case 3: CONV_AS(T, W, 3); break;      \
    case 4: CONV_AS(T, W, 4); break;      \
    case 5: CONV_AS(T, W, 5); break;      \
    default: CONV_AS(T, W, 0); break;     \
  }
  if (dtype == PAE_F32) {
    if (vec) { CONV_BY_TAPS(float, 4) } else { CONV_BY_TAPS(float, 1) }
  } else {
    if (vec) { CONV_BY_TAPS(bf16_t, 4) } else { CONV_BY_TAPS(bf16_t, 1) }
  }
#undef CONV_BY_TAPS
#undef CONV_AS
  return pae_check_launch("input_conv");
}

// Row t is the one token of sequence t, at positions[t], its ring in slot slots[t].  A thread owns up to four chunks of
// four channels; everything that does not depend on the norm (the branch, the stream, the ring, the filters) is asked for
// before the sum of squares is known.
template <typename T>
__global__ __launch_bounds__(256) void norm_join_conv_kernel(float* __restrict__ residual, const void* __restrict__ y, int parts,
                                                             int64_t part_stride, const void* __restrict__ weight,
                                                             int w_is_f32, float eps, float scale,
                                                             const float* __restrict__ filters, float* __restrict__ ring_base,
                                                             int64_t slot_stride, const int* __restrict__ positions,
                                                             const int* __restrict__ slots, int taps, T* __restrict__ rows,
                                                             int hidden) {
  __shared__ float scratch[4];
  const int t = blockIdx.x;
  const int64_t base = (int64_t)t * hidden;
  const int keep = taps - 1, pos = positions[t];
  float* ring = ring_base + (int64_t)slots[t] * slot_stride;
  const int nvec = hidden / 4;
  float yv[4][4], rv[4][4], past[4][4];  // the branch, the stream, the convolution's sum over the tokens before
  float ss = 0.f;
#pragma unroll
  for (int c = 0; c < 4; ++c) {
    const int v4 = threadIdx.x + 256 * c;
    if (v4 >= nvec) break;
    if (parts == 0) {
      if (sizeof(T) == 4) {
        conv_load<4>((const float*)y + base + 4 * v4, yv[c]);
      } else {
        const uint2 a = reinterpret_cast<const uint2*>((const bf16_t*)y + base)[v4];
        yv[c][0] = __uint_as_float(a.x << 16); yv[c][1] = __uint_as_float(a.x & 0xffff0000u);
        yv[c][2] = __uint_as_float(a.y << 16); yv[c][3] = __uint_as_float(a.y & 0xffff0000u);
      }
    } else {
      yv[c][0] = yv[c][1] = yv[c][2] = yv[c][3] = 0.f;
      for (int p = 0; p < parts; ++p) {  // partial sums are added in order
        float a[4];
        conv_load<4>((const float*)y + p * part_stride + base + 4 * v4, a);
#pragma unroll
        for (int i = 0; i < 4; ++i) yv[c][i] += a[i];
      }
    }
    conv_load<4>(residual + base + 4 * v4, rv[c]);
    past[c][0] = past[c][1] = past[c][2] = past[c][3] = 0.f;
    for (int j = 0; j < keep; ++j) {  // oldest first: tap j weighs the input keep - j tokens ago
      const int p = pos - keep + j;
      if (p < 0) continue;
      float w[4], in[4];
      conv_load<4>(filters + (int64_t)j * hidden + 4 * v4, w);
      conv_load<4>(ring + (int64_t)(p % keep) * hidden + 4 * v4, in);
#pragma unroll
      for (int i = 0; i < 4; ++i) past[c][i] = fmaf(w[i], in[i], past[c][i]);
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) ss = fmaf(yv[c][i], yv[c][i], ss);
  }
  const float total = block_sum<4>(ss, scratch);
  const float inv = 1.0f / sqrtf(total / (float)hidden + eps);
#pragma unroll
  for (int c = 0; c < 4; ++c) {
    const int v4 = threadIdx.x + 256 * c;
    if (v4 >= nvec) break;
    float r[4], v[4], w[4];
    conv_load<4>(filters + (int64_t)keep * hidden + 4 * v4, w);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      r[i] = rv[c][i] + scale * (yv[c][i] * inv * load_param(weight, w_is_f32, 4 * v4 + i));
      v[i] = r[i] + fmaf(w[i], r[i], past[c][i]);
    }
    *reinterpret_cast<float4*>(residual + base + 4 * v4) = make_float4(r[0], r[1], r[2], r[3]);
    if (keep > 0) *reinterpret_cast<float4*>(ring + (int64_t)(pos % keep) * hidden + 4 * v4) = make_float4(r[0], r[1], r[2], r[3]);
    conv_store<T, 4>(rows + base + 4 * v4, v);
  }
}

extern "C" int pae_norm_join_conv_supported(int hidden) { return hidden > 0 && hidden % 4 == 0 && hidden <= 4096; }

extern "C" int pae_norm_join_conv(int dtype, float* residual, const void* y, int parts, int64_t part_stride, const void* weight,
                                  int w_is_f32, float eps, float scale, const float* filters, float* ring, int64_t slot_stride,
                                  const int* positions, const int* slots, int taps, void* rows, int num_rows, int hidden,
                                  hipStream_t stream) {
  PAE_REQUIRE(pae_norm_join_conv_supported(hidden) && part_stride % 4 == 0 && slot_stride % 4 == 0,
              "norm, join and convolution: width %d is no multiple of four up to 4,096", hidden);
  PAE_REQUIRE(taps >= 1 && taps <= 64 && parts >= 0, "norm, join and convolution: %d taps, %d parts", taps, parts);
  PAE_REQUIRE(taps == 1 || (ring && slot_stride >= (int64_t)(taps - 1) * hidden), "norm, join and convolution: %d taps need the requests' state", taps);
  if (num_rows <= 0) return 0;
  if (dtype == PAE_F32)
    norm_join_conv_kernel<float><<<num_rows, 256, 0, stream>>>(residual, y, parts, part_stride, weight, w_is_f32, eps, scale,
                                                               filters, ring, slot_stride, positions, slots, taps, (float*)rows, hidden);
  else if (dtype == PAE_BF16)
    norm_join_conv_kernel<bf16_t><<<num_rows, 256, 0, stream>>>(residual, y, parts, part_stride, weight, w_is_f32, eps, scale,
                                                                filters, ring, slot_stride, positions, slots, taps, (bf16_t*)rows, hidden);
  else
    return pae_fail("norm, join and convolution: unknown dtype code %d", dtype);
  return pae_check_launch("norm_join_conv");
}
