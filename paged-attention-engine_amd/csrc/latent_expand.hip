// Latent attention over long runs of tokens with the heads' keys and values formed: where a run holds many queries, a
// key of D + rd features and a value of V cost the attention far less per query than one row of kv_rank + rd features that
// is key and value at once, and forming them is one product over the run's keys.  (Few queries read the cached rows as
// they are; see attention_latent.hip.)  Around that product:
//
//   latent_gather    the cached latents of every key of the runs, page by page of 16, as rows of a matrix [keys][rank];
//                    rows behind a run's last key are zero
//   latent_expand    the product's rows [H heads of D keys | H heads of V values] to pages of 16 keys: keys
//                    [page][H][16][KD] = [D features | the cached rotated part, rd | zeros], values transposed within
//                    the page, [page][H][V][16]
//   latent_queries   query heads [D | rd] of the projected rows to rows [H][KD] = [D | rd, the first `rot` rotated | zeros]
//
// pages[p] = (table row of the sequence, position of the page's first key, keys in the page, unused).
// bfloat16; the rotation is float32 and rounded once.
#include "common.h"
#include "api.h"

__global__ __launch_bounds__(256) void latent_gather_kernel(bf16_t* __restrict__ rows, const bf16_t* __restrict__ latent,
                                                            const int4* __restrict__ pages, const int* __restrict__ block_tables,
                                                            int max_blocks, int bs, int rank, int width) {
  const int4 page = pages[blockIdx.x];
  const int64_t block = block_tables[(int64_t)page.x * max_blocks + page.y / bs];
  const bf16_t* src = latent + (block * bs + page.y % bs) * (int64_t)width;
  bf16_t* dst = rows + (int64_t)blockIdx.x * 16 * rank;
  const int vecs = rank / 8;  // rank % 32 == 0, so rows start on 16-byte boundaries where width % 8 == 0 (checked by the caller)
  for (int e = threadIdx.x; e < 16 * vecs; e += 256) {
    const int j = e / vecs, v = e % vecs;
    uint4 x = make_uint4(0, 0, 0, 0);
    if (j < page.z) x = reinterpret_cast<const uint4*>(src + (int64_t)j * width)[v];
    reinterpret_cast<uint4*>(dst + (int64_t)j * rank)[v] = x;
  }
}

__global__ __launch_bounds__(256) void latent_expand_kernel(bf16_t* __restrict__ keys, bf16_t* __restrict__ values,
                                                            const bf16_t* __restrict__ up, int64_t up_stride,
                                                            const bf16_t* __restrict__ latent, const int4* __restrict__ pages,
                                                            const int* __restrict__ block_tables, int max_blocks, int bs, int H,
                                                            int D, int rd, int V, int rank, int KD) {
  extern __shared__ bf16_t tile[];  // [16][V + 2]: the page's values, to be written the other way round
  const int h = blockIdx.y;
  const int4 page = pages[blockIdx.x];
  const int width = rank + rd;
  const int64_t block = block_tables[(int64_t)page.x * max_blocks + page.y / bs];
  const bf16_t* cached = latent + (block * bs + page.y % bs) * (int64_t)width + rank;
  const bf16_t* src = up + (int64_t)blockIdx.x * 16 * up_stride;
  bf16_t* kd = keys + ((int64_t)blockIdx.x * H + h) * 16 * KD;
  const bf16_t zero = __float2bfloat16(0.f);
  for (int e = threadIdx.x; e < 8 * KD; e += 256) {  // two features a thread: D, rd and KD are even
    const int j = e / (KD / 2), d = e % (KD / 2) * 2;
    ushort2 x = make_ushort2(0, 0);
    if (j < page.z) {
      if (d < D) x = *reinterpret_cast<const ushort2*>(src + j * up_stride + h * D + d);
      else if (d < D + rd) x = *reinterpret_cast<const ushort2*>(cached + (int64_t)j * width + d - D);
    }
    *reinterpret_cast<ushort2*>(kd + j * KD + d) = x;
  }
  for (int e = threadIdx.x; e < 8 * V; e += 256) {
    const int j = e / (V / 2), v = e % (V / 2) * 2;
    const bf16_t* at = src + j * up_stride + (int64_t)H * D + h * V + v;
    tile[j * (V + 2) + v] = j < page.z ? at[0] : zero;
    tile[j * (V + 2) + v + 1] = j < page.z ? at[1] : zero;
  }
  __syncthreads();
  bf16_t* vd = values + ((int64_t)blockIdx.x * H + h) * V * 16;
  for (int e = threadIdx.x; e < 8 * V; e += 256) {
    const int v = e / 8, j = e % 8 * 2;
    vd[v * 16 + j] = tile[j * (V + 2) + v];
    vd[v * 16 + j + 1] = tile[(j + 1) * (V + 2) + v];
  }
}

__global__ __launch_bounds__(256) void latent_queries_kernel(bf16_t* __restrict__ out, const bf16_t* __restrict__ proj,
                                                             int64_t row_stride, const float* __restrict__ cos_sin,
                                                             float magnitude, int H, int D, int rd, int rot, int interleaved,
                                                             int KD) {
  const int64_t t = blockIdx.x;
  const bf16_t* row = proj + t * row_stride;
  bf16_t* dst = out + t * H * KD;
  const int half = rot / 2;
  for (int e = threadIdx.x; e < H * KD; e += 256) {
    const int h = e / KD, d = e % KD;
    const bf16_t* head = row + (int64_t)h * (D + rd);
    float x = 0.f;
    if (d >= D && d < D + rot) {
      const int i = d - D;
      const int pair = interleaved ? i / 2 : i % half;
      const int first = interleaved ? i % 2 == 0 : i < half;
      const int other = interleaved ? i ^ 1 : (i < half ? i + half : i - half);
      const float c = magnitude * cos_sin[(t * half + pair) * 2], s = magnitude * cos_sin[(t * half + pair) * 2 + 1];
      const float a = to_f32(head[D + i]), b = to_f32(head[D + other]);
      x = first ? a * c - b * s : a * c + b * s;
    } else if (d < D + rd) {
      x = to_f32(head[d]);
    }
    dst[e] = __float2bfloat16(x);
  }
}

extern "C" int pae_latent_gather(void* rows, const void* latent, const int* pages, int num_pages, const int* block_tables,
                                 int max_blocks, int bs, int rank, int width, hipStream_t stream) {
  PAE_REQUIRE(rank > 0 && rank % 8 == 0 && width >= rank && width % 8 == 0, "latent_gather: latent %d of rows of %d", rank, width);
  PAE_REQUIRE(bs >= 16 && bs % 16 == 0 && max_blocks > 0, "latent_gather: page size %d is not a multiple of 16", bs);
  if (num_pages <= 0) return 0;
  latent_gather_kernel<<<num_pages, 256, 0, stream>>>((bf16_t*)rows, (const bf16_t*)latent, (const int4*)pages, block_tables,
                                                      max_blocks, bs, rank, width);
  return pae_check_launch("latent_gather");
}

extern "C" int pae_latent_expand(void* keys, void* values, const void* up, int64_t up_stride, const void* latent,
                                 const int* pages, int num_pages, const int* block_tables, int max_blocks, int bs, int H, int D,
                                 int rd, int V, int rank, int KD, hipStream_t stream) {
  PAE_REQUIRE(H > 0 && H <= 65535 && D > 0 && rd >= 0 && V > 0 && rank > 0, "latent_expand: bad sizes H=%d D=%d rd=%d V=%d", H, D, rd, V);
  PAE_REQUIRE(D % 2 == 0 && rd % 2 == 0 && V % 2 == 0 && rank % 2 == 0 && KD % 2 == 0 && D + rd <= KD && V <= 1024,
              "latent_expand: keys of %d + %d in rows of %d, values of %d", D, rd, KD, V);
  PAE_REQUIRE(up_stride >= (int64_t)H * (D + V) && up_stride % 2 == 0, "latent_expand: row stride %lld too small", (long long)up_stride);
  PAE_REQUIRE(bs >= 16 && bs % 16 == 0 && max_blocks > 0, "latent_expand: page size %d is not a multiple of 16", bs);
  if (num_pages <= 0) return 0;
  latent_expand_kernel<<<dim3(num_pages, H), 256, 16 * (V + 2) * sizeof(bf16_t), stream>>>(
      (bf16_t*)keys, (bf16_t*)values, (const bf16_t*)up, up_stride, (const bf16_t*)latent, (const int4*)pages, block_tables,
      max_blocks, bs, H, D, rd, V, rank, KD);
  return pae_check_launch("latent_expand");
}

extern "C" int pae_latent_queries(void* out, const void* proj, int64_t row_stride, int num_tokens, const float* cos_sin,
                                  float magnitude, int H, int D, int rd, int rot, int interleaved, int KD, hipStream_t stream) {
  PAE_REQUIRE(H > 0 && D > 0 && rd >= 0 && D + rd <= KD && rot >= 0 && rot <= rd && rot % 2 == 0, "latent_queries: bad sizes");
  PAE_REQUIRE(rot == 0 || cos_sin, "latent_queries: a rotation needs its table of cosines and sines");
  PAE_REQUIRE(row_stride >= (int64_t)H * (D + rd), "latent_queries: row stride %lld too small", (long long)row_stride);
  if (num_tokens <= 0) return 0;
  latent_queries_kernel<<<num_tokens, 256, 0, stream>>>((bf16_t*)out, (const bf16_t*)proj, row_stride, cos_sin, magnitude, H, D,
                                                        rd, rot, interleaved, KD);
  return pae_check_launch("latent_queries");
}
