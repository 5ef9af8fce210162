// Linear attention with a fixed decay per head (lightning attention): a recurrent mixer whose per-request state is one
// matrix S [D, V] per head,
//
//   S_t = a_h S_(t-1) + k_t v_t^T;   o_t = S_t^T q_t,     q, k, v = act(projected rows), act SiLU or none
//
// then all heads' o are divided by their common root mean square, multiplied by a weight per feature and by
// act(gate) (sigmoid or SiLU) and rounded to the activation type.  A step's projected rows hold, per token,
// [q: H heads of D | k: H heads of D | v: H heads of V]; S lies in the request's slot as [H][V][D], float32.
//
// A request's run of a few tokens walks the recurrence token by token (serial).  Longer runs are cut into chunks of C
// tokens, and since the decay is one number per head, what a chunk does is three products in float32 on the matrix
// cores (v_mfma_f32_16x16x4_f32: products and sums in full 32-bit):
//
//   chunk_sums   K_c = sum_j a^(n-1-j) v_j k_j^T       what chunk c (of n tokens) adds to the state, every chunk at once
//   chunk_scan   S_c <- the state before chunk c;  S_(c+1) = a^n S_c + K_c      along the run, every element by itself
//   chunk_out    o_i = a^(i+1) S_c^T q_i + sum_(j <= i) a^(i-j) (k_j . q_i) v_j        every chunk at once
//
// Powers of the decay come from a table a^0 .. a^C formed in double precision.  All of it is float32; only the
// projected rows and the result are in the activation type.  A decay of 1, 0 or above 1 needs no special case.
#include "common.h"
#include "api.h"
#include "recurrent_device.h"

#define FD_VS 64  // value features of a workgroup in the chunk kernels

// ---------------------------------------------------------------------------------------------- serial
// runs[i] = (table row of the sequence, first flat row, rows, unused).  One workgroup per (run, head, 16 columns of S);
// a column's D rows are shared out over 16 lanes (rows 64 r + 4 lane + 0..3), which keep them in registers.
#define FD_STEPS 4  // tokens staged at a time
template <typename T, int R>
__global__ __launch_bounds__(256) void fixed_decay_serial_kernel(const T* __restrict__ proj, int64_t row_stride,
                                                                 const int4* __restrict__ runs, const int* __restrict__ slots,
                                                                 float* __restrict__ state, int64_t slot_stride,
                                                                 const float* __restrict__ powers, int power_stride, int H,
                                                                 int D, int V, int silu, float* __restrict__ out) {
  __shared__ __attribute__((aligned(16))) float s_k[FD_STEPS * R * 64];
  __shared__ __attribute__((aligned(16))) float s_q[FD_STEPS * R * 64];
  constexpr int DP = R * 64;
  const int4 run = runs[blockIdx.x];
  const int h = blockIdx.y;
  const int col = blockIdx.z * 16 + threadIdx.x / 16, sub = threadIdx.x % 16;
  const bool live = col < V;
  const bool vec = D % 4 == 0;
  const float decay = powers[(int64_t)h * power_stride + 1];
  float* column = state + (int64_t)slots[run.x] * slot_stride + ((int64_t)h * V + (live ? col : 0)) * D;
  float S[R][4];
#pragma unroll
  for (int r = 0; r < R; ++r) {
    const int d = 64 * r + 4 * sub;
    if (live && vec && d < D) {
      const float4 x = *reinterpret_cast<const float4*>(column + d);
      S[r][0] = x.x; S[r][1] = x.y; S[r][2] = x.z; S[r][3] = x.w;
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e) S[r][e] = live && d + e < D ? column[d + e] : 0.f;
    }
  }
  const bool rows_vec = vec && row_stride % 4 == 0 && (uintptr_t)proj % 16 == 0;
  for (int first = 0; first < run.z; first += FD_STEPS) {
    const int n = min(FD_STEPS, run.z - first);
    __syncthreads();  // the tokens before have been worked through
    for (int e = threadIdx.x; e < n * 2 * (DP / 4); e += 256) {
      const int which = e / (DP / 4), d = e % (DP / 4) * 4, i = which / 2;
      const T* row = proj + (int64_t)(run.y + first + i) * row_stride + ((which % 2) * H + h) * (int64_t)D;
      float x[4];
      load_row4(row, d, D, rows_vec, silu, x);
      *reinterpret_cast<float4*>((which % 2 ? s_k : s_q) + i * DP + d) = make_float4(x[0], x[1], x[2], x[3]);
    }
    float v[FD_STEPS];
#pragma unroll
    for (int i = 0; i < FD_STEPS; ++i)
      v[i] = i < n && live ? recurrent_act(to_f32(proj[(int64_t)(run.y + first + i) * row_stride + 2 * H * (int64_t)D + h * V + col]), silu) : 0.f;
    __syncthreads();
#pragma unroll
    for (int i = 0; i < FD_STEPS; ++i) {
      if (i >= n) break;
      float o = 0.f;
#pragma unroll
      for (int r = 0; r < R; ++r) {
        const float4 k4 = *reinterpret_cast<const float4*>(s_k + i * DP + 64 * r + 4 * sub);
        const float4 q4 = *reinterpret_cast<const float4*>(s_q + i * DP + 64 * r + 4 * sub);
        S[r][0] = fmaf(k4.x, v[i], decay * S[r][0]); o = fmaf(S[r][0], q4.x, o);
        S[r][1] = fmaf(k4.y, v[i], decay * S[r][1]); o = fmaf(S[r][1], q4.y, o);
        S[r][2] = fmaf(k4.z, v[i], decay * S[r][2]); o = fmaf(S[r][2], q4.z, o);
        S[r][3] = fmaf(k4.w, v[i], decay * S[r][3]); o = fmaf(S[r][3], q4.w, o);
      }
      o = sum16(o);
      if (live && sub == 0) out[((int64_t)(run.y + first + i) * H + h) * V + col] = o;
    }
  }
  if (!live) return;
#pragma unroll
  for (int r = 0; r < R; ++r) {
    const int d = 64 * r + 4 * sub;
    if (vec && d < D) {
      *reinterpret_cast<float4*>(column + d) = make_float4(S[r][0], S[r][1], S[r][2], S[r][3]);
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (d + e < D) column[d + e] = S[r][e];
    }
  }
}

// ---------------------------------------------------------------------------------------------- chunks
// chunks[c] = (table row of the sequence, first flat row, rows n <= C, unused).  One workgroup (C / 16 wavefronts) per
// (chunk, head, FD_VS value features): sums [chunk][H][V][D].
template <typename T, int DT, int C>
__global__ __launch_bounds__(C * 4) void fixed_decay_chunk_sums_kernel(const T* __restrict__ proj, int64_t row_stride,
                                                                       const int4* __restrict__ chunks,
                                                                       const float* __restrict__ powers, int H, int D, int V,
                                                                       int silu, float* __restrict__ sums) {
  constexpr int NT = C * 4, DS = DT * 16 + 4, VST = FD_VS + 4;
  __shared__ __attribute__((aligned(16))) float s_k[C * DS];
  __shared__ __attribute__((aligned(16))) float s_v[C * VST];
  const int4 chunk = chunks[blockIdx.x];
  const int h = blockIdx.y, v0 = blockIdx.z * FD_VS;
  const int n = chunk.z;
  const float* pw = powers + (int64_t)h * (C + 1);
  const bool aligned = row_stride % 4 == 0 && (uintptr_t)proj % 16 == 0;
  const bool kvec = aligned && D % 4 == 0, vvec = aligned && V % 4 == 0 && 2 * H * D % 4 == 0;
  for (int e = threadIdx.x; e < C * DT * 4; e += NT) {
    const int j = e / (DT * 4), d = e % (DT * 4) * 4;
    float x[4] = {0.f, 0.f, 0.f, 0.f};
    if (j < n) {
      load_row4(proj + (int64_t)(chunk.y + j) * row_stride + (H + h) * (int64_t)D, d, D, kvec, silu, x);
      const float w = pw[n - 1 - j];
#pragma unroll
      for (int i = 0; i < 4; ++i) x[i] *= w;
    }
    *reinterpret_cast<float4*>(s_k + j * DS + d) = make_float4(x[0], x[1], x[2], x[3]);
  }
  for (int e = threadIdx.x; e < C * (FD_VS / 4); e += NT) {
    const int j = e / (FD_VS / 4), v = e % (FD_VS / 4) * 4;
    float x[4] = {0.f, 0.f, 0.f, 0.f};
    if (j < n && v0 + v < V)
      load_row4(proj + (int64_t)(chunk.y + j) * row_stride + 2 * H * (int64_t)D + h * V, v0 + v, V, vvec, silu, x);
    *reinterpret_cast<float4*>(s_v + j * VST + v) = make_float4(x[0], x[1], x[2], x[3]);
  }
  __syncthreads();
  const int lane = threadIdx.x % PAE_WAVE, wave = threadIdx.x / PAE_WAVE, col = lane % 16, g4 = lane / 16;
  float* dst = sums + ((int64_t)blockIdx.x * H + h) * V * D;
  for (int dt = wave; dt < DT; dt += C / 16) {
    if (dt * 16 >= D) break;
    f32x4 acc[FD_VS / 16];
#pragma unroll
    for (int vt = 0; vt < FD_VS / 16; ++vt) acc[vt] = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int s = 0; s < C / 4; ++s) {
      const int j = 4 * s + g4;
      const float b = s_k[j * DS + dt * 16 + col];
#pragma unroll
      for (int vt = 0; vt < FD_VS / 16; ++vt)
        acc[vt] = __builtin_amdgcn_mfma_f32_16x16x4f32(s_v[j * VST + vt * 16 + col], b, acc[vt], 0, 0, 0);
    }
    const int d = dt * 16 + col;
    if (d < D) {
#pragma unroll
      for (int vt = 0; vt < FD_VS / 16; ++vt)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int v = v0 + vt * 16 + 4 * g4 + i;
          if (v < V) dst[(int64_t)v * D + d] = acc[vt][i];
        }
    }
  }
}

// scans[s] = (table row of the sequence, its first chunk, its chunks, rows of its last chunk; all others hold C).  A thread
// per element of the state: sums become the states before every chunk, and the slot receives the state after the last.
template <int C>
__global__ __launch_bounds__(256) void fixed_decay_chunk_scan_kernel(float* __restrict__ sums, const int4* __restrict__ scans,
                                                                     const int* __restrict__ slots, float* __restrict__ state,
                                                                     int64_t slot_stride, const float* __restrict__ powers,
                                                                     int64_t per_head, int64_t total) {
  const int64_t e = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (e >= total) return;
  const int4 scan = scans[blockIdx.y];
  const float* pw = powers + e / per_head * (C + 1);
  const float full = pw[C], last = pw[scan.w];
  float* held = state + (int64_t)slots[scan.x] * slot_stride + e;
  float* at = sums + (int64_t)scan.y * total + e;
  float S = *held;
  constexpr int AHEAD = 8;
  for (int c0 = 0; c0 < scan.z; c0 += AHEAD) {
    float added[AHEAD];
#pragma unroll
    for (int i = 0; i < AHEAD; ++i) added[i] = c0 + i < scan.z ? at[(c0 + i) * total] : 0.f;
#pragma unroll
    for (int i = 0; i < AHEAD; ++i) {
      if (c0 + i >= scan.z) break;
      at[(c0 + i) * total] = S;
      S = fmaf(c0 + i + 1 == scan.z ? last : full, S, added[i]);
    }
  }
  *held = S;
}

// One workgroup per (chunk, head, FD_VS value features); wavefront w has the queries 16 w .. 16 w + 15.  The scores are
// formed as K Q^T, whose accumulator (row = key 4 g4 + i, column = query) is the second product's B operand as it is.
template <typename T, int DT, int C>
__global__ __launch_bounds__(C * 4) void fixed_decay_chunk_out_kernel(const T* __restrict__ proj, int64_t row_stride,
                                                                      const int4* __restrict__ chunks,
                                                                      const float* __restrict__ powers, int H, int D, int V,
                                                                      int silu, const float* __restrict__ before,
                                                                      float* __restrict__ out) {
  constexpr int NT = C * 4, DS = DT * 16 + 4, VST = FD_VS + 4;
  __shared__ __attribute__((aligned(16))) float s_k[C * DS];
  __shared__ __attribute__((aligned(16))) float s_v[C * VST];
  __shared__ float s_pw[C + 1];
  const int4 chunk = chunks[blockIdx.x];
  const int h = blockIdx.y, v0 = blockIdx.z * FD_VS;
  const int n = chunk.z;
  const bool aligned = row_stride % 4 == 0 && (uintptr_t)proj % 16 == 0;
  const bool kvec = aligned && D % 4 == 0, vvec = aligned && V % 4 == 0 && 2 * H * D % 4 == 0;
  const int lane = threadIdx.x % PAE_WAVE, wave = threadIdx.x / PAE_WAVE, col = lane % 16, g4 = lane / 16;
  const int query = wave * 16 + col;  // this lane's query within the chunk
  float q[DT][4];                      // features 16 s + 4 g4 + i of it
#pragma unroll
  for (int s = 0; s < DT; ++s) {
#pragma unroll
    for (int i = 0; i < 4; ++i) q[s][i] = 0.f;
    if (query < n) load_row4(proj + (int64_t)(chunk.y + query) * row_stride + h * (int64_t)D, 16 * s + 4 * g4, D, kvec, silu, q[s]);
  }
  for (int e = threadIdx.x; e < C * DT * 4; e += NT) {
    const int j = e / (DT * 4), d = e % (DT * 4) * 4;
    float x[4] = {0.f, 0.f, 0.f, 0.f};
    if (j < n) load_row4(proj + (int64_t)(chunk.y + j) * row_stride + (H + h) * (int64_t)D, d, D, kvec, silu, x);
    *reinterpret_cast<float4*>(s_k + j * DS + d) = make_float4(x[0], x[1], x[2], x[3]);
  }
  for (int e = threadIdx.x; e < C * (FD_VS / 4); e += NT) {
    const int j = e / (FD_VS / 4), v = e % (FD_VS / 4) * 4;
    float x[4] = {0.f, 0.f, 0.f, 0.f};
    if (j < n && v0 + v < V)
      load_row4(proj + (int64_t)(chunk.y + j) * row_stride + 2 * H * (int64_t)D + h * V, v0 + v, V, vvec, silu, x);
    *reinterpret_cast<float4*>(s_v + j * VST + v) = make_float4(x[0], x[1], x[2], x[3]);
  }
  if (threadIdx.x <= C) s_pw[threadIdx.x] = powers[(int64_t)h * (C + 1) + threadIdx.x];
  __syncthreads();
  if (wave * 16 >= n) return;  // no barrier follows
  f32x4 acc[FD_VS / 16];
#pragma unroll
  for (int vt = 0; vt < FD_VS / 16; ++vt) acc[vt] = (f32x4){0.f, 0.f, 0.f, 0.f};
  // what the state before the chunk holds for these queries
  const float* S = before + ((int64_t)blockIdx.x * H + h) * V * D;
  const bool svec = D % 4 == 0;
#pragma unroll
  for (int s = 0; s < DT; ++s) {
    const int d = 16 * s + 4 * g4;
    if (16 * s >= D) break;
    float sv[FD_VS / 16][4];
#pragma unroll
    for (int vt = 0; vt < FD_VS / 16; ++vt) {
      const int v = v0 + vt * 16 + col;
      if (svec && v < V && d < D) {
        const float4 x = *reinterpret_cast<const float4*>(S + (int64_t)v * D + d);
        sv[vt][0] = x.x; sv[vt][1] = x.y; sv[vt][2] = x.z; sv[vt][3] = x.w;
      } else {
#pragma unroll
        for (int i = 0; i < 4; ++i) sv[vt][i] = v < V && d + i < D ? S[(int64_t)v * D + d + i] : 0.f;
      }
    }
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int vt = 0; vt < FD_VS / 16; ++vt)
        acc[vt] = __builtin_amdgcn_mfma_f32_16x16x4f32(sv[vt][i], q[s][i], acc[vt], 0, 0, 0);
  }
  const float reach = s_pw[query + 1];
#pragma unroll
  for (int vt = 0; vt < FD_VS / 16; ++vt)
#pragma unroll
    for (int i = 0; i < 4; ++i) acc[vt][i] *= reach;
  // the chunk's own keys up to the query
  for (int jt = 0; jt <= wave; ++jt) {
    f32x4 p = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int s = 0; s < DT; ++s) {
      const float4 k4 = *reinterpret_cast<const float4*>(s_k + (jt * 16 + col) * DS + 16 * s + 4 * g4);
      p = __builtin_amdgcn_mfma_f32_16x16x4f32(k4.x, q[s][0], p, 0, 0, 0);
      p = __builtin_amdgcn_mfma_f32_16x16x4f32(k4.y, q[s][1], p, 0, 0, 0);
      p = __builtin_amdgcn_mfma_f32_16x16x4f32(k4.z, q[s][2], p, 0, 0, 0);
      p = __builtin_amdgcn_mfma_f32_16x16x4f32(k4.w, q[s][3], p, 0, 0, 0);
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int back = query - (jt * 16 + 4 * g4 + i);
      p[i] = back >= 0 ? p[i] * s_pw[back] : 0.f;
    }
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int vt = 0; vt < FD_VS / 16; ++vt)
        acc[vt] = __builtin_amdgcn_mfma_f32_16x16x4f32(s_v[(jt * 16 + 4 * g4 + i) * VST + vt * 16 + col], p[i], acc[vt], 0, 0, 0);
  }
  if (query >= n) return;
  float* dst = out + ((int64_t)(chunk.y + query) * H + h) * V;
#pragma unroll
  for (int vt = 0; vt < FD_VS / 16; ++vt) {
    const int v = v0 + vt * 16 + 4 * g4;
    if (V % 4 == 0 && v < V) {
      *reinterpret_cast<float4*>(dst + v) = make_float4(acc[vt][0], acc[vt][1], acc[vt][2], acc[vt][3]);
    } else {
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (v + i < V) dst[v + i] = acc[vt][i];
    }
  }
}

// ---------------------------------------------------------------------------------------------- norm and gate
// out[t] = T(x[t] / sqrt(mean(x[t]^2) + eps) * w * act(gate[t])) over the whole row of N features.
template <typename T, bool VEC>
__global__ __launch_bounds__(256) void row_norm_gate_kernel(const float* __restrict__ x, const T* __restrict__ gates,
                                                            int64_t gate_stride, int gate_sigmoid,
                                                            const void* __restrict__ weight, int w_is_f32, float eps, int N,
                                                            T* __restrict__ out) {
  __shared__ float scratch[4];
  const int64_t t = blockIdx.x;
  const float* row = x + t * N;
  const T* gate = gates + t * gate_stride;
  T* dst = out + t * N;
  constexpr int W = VEC ? 4 : 1;
  float ss = 0.f;
  for (int i = threadIdx.x * W; i < N; i += 256 * W) {
    if (VEC) {
      const float4 a = *reinterpret_cast<const float4*>(row + i);
      ss = fmaf(a.x, a.x, ss); ss = fmaf(a.y, a.y, ss); ss = fmaf(a.z, a.z, ss); ss = fmaf(a.w, a.w, ss);
    } else {
      ss = fmaf(row[i], row[i], ss);
    }
  }
  ss = block_sum<4>(ss, scratch);
  const float inv = 1.0f / sqrtf(ss / (float)N + eps);
  for (int i = threadIdx.x * W; i < N; i += 256 * W) {
    float z[4], r[4];
    if (VEC) {
      load_row4(gate, i, N, true, 0, z);
      const float4 a = *reinterpret_cast<const float4*>(row + i);
      r[0] = a.x; r[1] = a.y; r[2] = a.z; r[3] = a.w;
    } else {
      z[0] = to_f32(gate[i]);
      r[0] = row[i];
    }
#pragma unroll
    for (int e = 0; e < W; ++e) {
      const float sig = 1.0f / (1.0f + expf(-z[e]));
      r[e] = r[e] * inv * load_param(weight, w_is_f32, i + e) * (gate_sigmoid ? sig : z[e] * sig);
    }
    if (VEC && sizeof(T) == 4) {
      *reinterpret_cast<float4*>((float*)dst + i) = make_float4(r[0], r[1], r[2], r[3]);
    } else if (VEC) {
      bf16_t b[4] = {__float2bfloat16(r[0]), __float2bfloat16(r[1]), __float2bfloat16(r[2]), __float2bfloat16(r[3])};
      *reinterpret_cast<uint2*>((bf16_t*)dst + i) = *reinterpret_cast<const uint2*>(b);
    } else {
      dst[i] = from_f32<T>(r[0]);
    }
  }
}

// Tokens a chunk for key width D; 0: such heads take the serial kernel for runs of any length.
extern "C" int pae_fixed_decay_chunk(int D) { return D <= 128 ? 64 : (D <= 256 ? 32 : 0); }

template <typename T>
static int fixed_decay_launch(const T* proj, int64_t row_stride, const int4* serial, int num_serial, const int4* chunks,
                              int num_chunks, const int4* scans, int num_scans, const int* slots, const float* powers, int H,
                              int D, int V, int silu, float* state, int64_t slot_stride, float* sums, float* o,
                              hipStream_t stream) {
  const int chunk = pae_fixed_decay_chunk(D);
  if (num_serial > 0) {
    dim3 grid(num_serial, H, (V + 15) / 16);
    const int power_stride = (chunk ? chunk : 1) + 1;
#define FD_SERIAL(R)                                                                                                      \
  fixed_decay_serial_kernel<T, R><<<grid, 256, 0, stream>>>(proj, row_stride, serial, slots, state, slot_stride, powers, \
                                                            power_stride, H, D, V, silu, o)
    if (D <= 64) FD_SERIAL(1);
    else if (D <= 128) FD_SERIAL(2);
    else if (D <= 256) FD_SERIAL(4);
    else if (D <= 512) FD_SERIAL(8);
    else FD_SERIAL(16);
#undef FD_SERIAL
  }
  if (num_chunks > 0) {
    dim3 grid(num_chunks, H, (V + FD_VS - 1) / FD_VS);
    const int64_t total = (int64_t)H * V * D;
    dim3 scan_grid((unsigned)((total + 255) / 256), num_scans);
#define FD_CHUNKS(DT, C)                                                                                                  \
  do {                                                                                                                    \
    fixed_decay_chunk_sums_kernel<T, DT, C><<<grid, C * 4, 0, stream>>>(proj, row_stride, chunks, powers, H, D, V, silu, sums); \
    fixed_decay_chunk_scan_kernel<C><<<scan_grid, 256, 0, stream>>>(sums, scans, slots, state, slot_stride, powers,       \
                                                                    (int64_t)V * D, total);                              \
    fixed_decay_chunk_out_kernel<T, DT, C><<<grid, C * 4, 0, stream>>>(proj, row_stride, chunks, powers, H, D, V, silu,   \
                                                                       sums, o);                                          \
  } while (0)
    if (D <= 64) FD_CHUNKS(4, 64);
    else if (D <= 128) FD_CHUNKS(8, 64);
    else FD_CHUNKS(16, 32);
#undef FD_CHUNKS
  }
  return 0;
}

// `serial` int32 [num_serial][4], `chunks` [num_chunks][4], `scans` [num_scans][4] as the kernels above read them: between
// them they cover every row of the step once, a sequence in one of the lists only.  `powers` [H][C + 1] (C 1 where there
// are no chunks).  work: o [T][H V], then sums [num_chunks][H][V][D], each from a 16-byte boundary on.
extern "C" int pae_fixed_decay_step(int dtype, const void* proj, int64_t row_stride, const void* gate_in, int64_t gate_stride,
                                    int gate_sigmoid, int silu, int num_tokens, const int* serial, int num_serial,
                                    const int* chunks, int num_chunks, const int* scans, int num_scans, const int* slots,
                                    const float* powers, int H, int D, int V, float* state, int64_t slot_stride,
                                    const void* norm_w, int w_is_f32, float norm_eps, float* work, void* out,
                                    hipStream_t stream) {
  PAE_REQUIRE(H > 0 && D > 0 && V > 0, "fixed-decay attention: bad head sizes H=%d D=%d V=%d", H, D, V);
  PAE_REQUIRE(D <= 1024, "fixed-decay attention: key width %d exceeds 1024", D);
  PAE_REQUIRE(H <= 65535 && V <= 65535 && num_scans <= 65535, "fixed-decay attention: %d heads, %d value features, %d runs exceed the grid",
              H, V, num_scans);
  PAE_REQUIRE(row_stride >= 2 * (int64_t)H * D + (int64_t)H * V, "fixed-decay attention: row stride %lld too small", (long long)row_stride);
  PAE_REQUIRE(gate_in && gate_stride >= (int64_t)H * V, "fixed-decay attention: the gate's rows are missing or too narrow");
  PAE_REQUIRE(num_chunks == 0 || pae_fixed_decay_chunk(D) > 0, "fixed-decay attention: key width %d has no chunks", D);
  PAE_REQUIRE((num_chunks == 0) == (num_scans == 0), "fixed-decay attention: %d chunks with %d runs", num_chunks, num_scans);
  PAE_REQUIRE(dtype == PAE_F32 || dtype == PAE_BF16, "fixed-decay attention: unknown dtype code %d", dtype);
  if (num_tokens <= 0) return 0;
  const int N = H * V;
  float* o = work;
  float* sums = work + ((int64_t)num_tokens * N + 3) / 4 * 4;
#define FD_STEP(T)                                                                                                       \
  do {                                                                                                                   \
    fixed_decay_launch<T>((const T*)proj, row_stride, (const int4*)serial, num_serial, (const int4*)chunks, num_chunks,  \
                          (const int4*)scans, num_scans, slots, powers, H, D, V, silu, state, slot_stride, sums, o, stream); \
    if (N % 4 == 0 && gate_stride % 4 == 0 && (uintptr_t)gate_in % (4 * sizeof(T)) == 0 && (uintptr_t)out % (4 * sizeof(T)) == 0) \
      row_norm_gate_kernel<T, true><<<num_tokens, 256, 0, stream>>>(o, (const T*)gate_in, gate_stride, gate_sigmoid,      \
                                                                    norm_w, w_is_f32, norm_eps, N, (T*)out);             \
    else                                                                                                                 \
      row_norm_gate_kernel<T, false><<<num_tokens, 256, 0, stream>>>(o, (const T*)gate_in, gate_stride, gate_sigmoid,     \
                                                                     norm_w, w_is_f32, norm_eps, N, (T*)out);            \
  } while (0)
  if (dtype == PAE_F32) FD_STEP(float);
  else FD_STEP(bf16_t);
#undef FD_STEP
  return pae_check_launch("fixed_decay_step");
}

// floats of `work` that pae_fixed_decay_step needs
extern "C" int64_t pae_fixed_decay_work_floats(int num_tokens, int num_chunks, int H, int D, int V) {
  return ((int64_t)num_tokens * H * V + 3) / 4 * 4 + (int64_t)num_chunks * H * V * D;
}
