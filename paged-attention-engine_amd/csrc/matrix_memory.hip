// A matrix memory with exponential gates: a recurrent mixer whose per-request state is, per head, a matrix
// C [D, V], the sum of its gated keys n [D] and a running maximum m of the gates' logarithms.
//
// A step's projected rows hold, per token, [q: H heads of D | k: H heads of D | v: H heads of V].  With cap c and the
// float32 sums z of the two gate projections with their biases:
//
//   i = c tanh(z_i / c);   f = logsigmoid(c tanh(z_f / c));   m_t = max(f + m_(t-1), i)
//   keep = exp(f + m_(t-1) - m_t);   take = exp(i - m_t)
//   C <- keep C + take k v^T;   n <- keep n + take k
//   o = C^T q / (max(|n . q|, exp(-m_t)) + floor_eps),  q times D^-1/2
//
// then o is divided by its root mean square over V, multiplied by a weight (one per head and feature) and by
// sigmoid(gate), and rounded to the activation type.  m starts at 0 like C and n (a slot is zeroed when
// a request takes it).  The state lies in the request's slot as [H][V + 1][D], row V of a head being n: the memory's
// column for a value that is 1 for every token.
//
// Runs of a few tokens walk the recurrence (serial).  Longer runs are cut into chunks of CH tokens.  With the maxima
// known, what token j leaves for token t of its chunk is take_j times the product of the keeps after j, so a chunk is
// three products in float32 on the matrix cores (v_mfma_f32_16x16x4_f32: products and sums in full 32-bit):
//
//   memory_gates   the maxima of a whole run by a scan of the maps m -> max(f + m, i), which compose; per token take,
//                  exp(-m), and the logarithm of the product of the keeps since the chunk's first token
//   chunk_sums     what a chunk adds to the state, referred to the maximum at its end; every chunk at once
//   chunk_scan     the states before every chunk, along the run, every element by itself
//   chunk_out      the state before the chunk and the chunk's own tokens read by every query; every chunk at once
//   memory_finish  the division, the norm over V, weight and gate
//
// A keep's logarithm is f + m_(t-1) - m_t with the maxima as they are stored (float32), so that state and maximum
// always belong together; its sums over a chunk are formed in double precision and kept as two floats, and the
// difference of two of them is as exact as a float32 number can be, however long the chunk's decay is.  Everything but
// the projected rows and the gate's rows is float32 or better.
#include "common.h"
#include "api.h"
#include "recurrent_device.h"

#define MM_VS 64     // value features of a workgroup in the chunk kernels
#define MM_STEPS 4   // tokens the serial kernel stages at a time
#define MM_FEW 16    // tokens the serial gates take at a time

__device__ __forceinline__ float log_sigmoid_f(float z) { return fminf(z, 0.f) - log1pf(expf(-fabsf(z))); }

// Per token and head, [T][H] each: what the kernels below hand on.
struct MemoryGates {
  float* take;    // exp(i - m_t)
  float* floors;  // exp(-m_t)
  float* keep;    // serial runs: exp(f + m_(t-1) - m_t)
  float* reach;   // runs in chunks: the product of the keeps from the chunk's first token to this one, ...
  float* log_hi;  // ... and its logarithm in two parts
  float* log_lo;
};

// ---------------------------------------------------------------------------------------------- gates, few tokens
// runs[i] = (table row of the sequence, first flat row, rows, unused); one workgroup of four wavefronts per (run, head).
// Without `gate_logits` the two sums of every token are formed here from the mixer's input: a wavefront a sum.
template <typename T>
__global__ __launch_bounds__(256) void memory_gates_few_kernel(const float* __restrict__ gate_logits, const T* __restrict__ x,
                                                               int64_t ldx, const T* __restrict__ gate_w,
                                                               const float* __restrict__ gate_b, int hidden, int wide,
                                                               const int4* __restrict__ runs, const int* __restrict__ slots,
                                                               float* __restrict__ maximum, int64_t max_slot_stride, int H,
                                                               float cap, MemoryGates gates) {
  constexpr int VEC = 16 / sizeof(T);
  struct alignas(16) Chunk { T v[VEC]; };
  __shared__ float s_log[2][MM_FEW];  // the gates' logarithms: input, forget
  const int4 run = runs[blockIdx.x];
  const int h = blockIdx.y, wave = threadIdx.x / PAE_WAVE, lane = threadIdx.x % PAE_WAVE;
  float* m_at = maximum + (int64_t)slots[run.x] * max_slot_stride + h;
  float m = *m_at;
  for (int first = 0; first < run.z; first += MM_FEW) {
    const int n = min(MM_FEW, run.z - first);
    for (int u = wave; u < 2 * n; u += 4) {
      const int which = u % 2, j = u / 2;
      const int64_t t = run.y + first + j;
      float z = 0.f;
      if (gate_logits) {
        z = gate_logits[t * 2 * H + which * H + h];
      } else {
        const T* row = x + t * ldx;
        const T* w = gate_w + (int64_t)(which * H + h) * hidden;
        if (wide) {
          for (int k = lane * VEC; k < hidden; k += PAE_WAVE * VEC) {
            const Chunk a = *reinterpret_cast<const Chunk*>(row + k);
            const Chunk b = *reinterpret_cast<const Chunk*>(w + k);
#pragma unroll
            for (int e = 0; e < VEC; ++e) z = fmaf(to_f32(a.v[e]), to_f32(b.v[e]), z);
          }
        } else {
          for (int k = lane; k < hidden; k += PAE_WAVE) z = fmaf(to_f32(row[k]), to_f32(w[k]), z);
        }
        z = wave_sum(z) + gate_b[which * H + h];
      }
      z = cap * tanhf(z / cap);
      if (lane == 0) s_log[which][j] = which ? log_sigmoid_f(z) : z;
    }
    __syncthreads();
    for (int j = 0; j < n; ++j) {
      const float li = s_log[0][j], lf = s_log[1][j];
      const float next = fmaxf(lf + m, li);
      if (threadIdx.x == j) {
        const int64_t at = (int64_t)(run.y + first + j) * H + h;
        gates.keep[at] = expf(lf + m - next);
        gates.take[at] = expf(li - next);
        gates.floors[at] = expf(-next);
      }
      m = next;
    }
    __syncthreads();
  }
  if (threadIdx.x == 0) *m_at = m;
}

// ---------------------------------------------------------------------------------------------- gates, runs in chunks
// scans[s] = (table row of the sequence, its first chunk, its chunks, rows of its last chunk; all others hold CH).  One
// workgroup of 1,024 threads per (run, head), a thread a token.  Token t is the map m -> max(f + m, i); a wavefront
// composes its 64 maps by a scan, the wavefronts' maps are composed in order.
template <int CH>
__global__ __launch_bounds__(1024) void memory_gates_scan_kernel(const float* __restrict__ gate_logits, const int4* __restrict__ chunks,
                                                                 const int4* __restrict__ scans, const int* __restrict__ slots,
                                                                 float* __restrict__ maximum, int64_t max_slot_stride, int H,
                                                                 float cap, MemoryGates gates) {
  __shared__ double s_add[16], s_top[16];  // a wavefront's map: m -> max(s_add + m, s_top)
  __shared__ float s_last;
  const int4 scan = scans[blockIdx.y];
  const int h = blockIdx.x, lane = threadIdx.x % PAE_WAVE, wave = threadIdx.x / PAE_WAVE;
  const int first_row = chunks[scan.y].y, total = (scan.z - 1) * CH + scan.w;
  float* m_at = maximum + (int64_t)slots[scan.x] * max_slot_stride + h;
  float m0 = *m_at;
  for (int base = 0; base < total; base += 1024) {
    const int i = base + (int)threadIdx.x;
    const bool live = i < total;
    const int64_t t = first_row + i;
    float li = -INFINITY, lf = 0.f;  // a row past the end: the map that changes nothing
    if (live) {
      li = cap * tanhf(gate_logits[t * 2 * H + h] / cap);
      lf = log_sigmoid_f(cap * tanhf(gate_logits[t * 2 * H + H + h] / cap));
    }
    double add = lf, top = li;
#pragma unroll
    for (int off = 1; off < PAE_WAVE; off *= 2) {
      const double add_before = __shfl_up(add, off, PAE_WAVE), top_before = __shfl_up(top, off, PAE_WAVE);
      if (lane >= off) {
        top = fmax(top_before + add, top);
        add = add_before + add;
      }
    }
    if (lane == PAE_WAVE - 1) {
      s_add[wave] = add;
      s_top[wave] = top;
    }
    __syncthreads();
    double m_in = m0;  // before this wavefront's first token
    for (int w = 0; w < wave; ++w) m_in = fmax(s_add[w] + m_in, s_top[w]);
    const float after = (float)fmax(add + m_in, top);
    float before = __shfl_up(after, 1, PAE_WAVE);
    if (lane == 0) before = (float)m_in;
    double keeps = (double)lf + (double)before - (double)after;  // a keep's logarithm, then their sums within the chunk
#pragma unroll
    for (int off = 1; off < CH; off *= 2) {
      const double sum_before = __shfl_up(keeps, off, CH);
      if (lane % CH >= off) keeps += sum_before;
    }
    if (live) {
      const int64_t at = t * H + h;
      const float hi = (float)keeps;
      gates.log_hi[at] = hi;
      gates.log_lo[at] = (float)(keeps - (double)hi);
      gates.reach[at] = expf(hi);
      gates.take[at] = expf(li - after);
      gates.floors[at] = expf(-after);
    }
    if (i == min(base + 1024, total) - 1) s_last = after;
    __syncthreads();
    m0 = s_last;
  }
  if (threadIdx.x == 0) *m_at = m0;
}

// ---------------------------------------------------------------------------------------------- serial
// One workgroup per (run, head, 16 columns of the memory, column V being n); a column's D rows are shared out over 16
// lanes (rows 64 r + 4 lane + 0..3), which keep them in registers over the run.
template <typename T, int R>
__global__ __launch_bounds__(256) void memory_serial_kernel(const T* __restrict__ proj, int64_t row_stride,
                                                            const int4* __restrict__ runs, const int* __restrict__ slots,
                                                            float* __restrict__ state, int64_t slot_stride, MemoryGates gates,
                                                            int H, int D, int V, float* __restrict__ out, float* __restrict__ nq) {
  constexpr int DP = R * 64;
  __shared__ __attribute__((aligned(16))) float s_k[MM_STEPS * DP];
  __shared__ __attribute__((aligned(16))) float s_q[MM_STEPS * DP];
  const int4 run = runs[blockIdx.x];
  const int h = blockIdx.y;
  const int col = blockIdx.z * 16 + threadIdx.x / 16, sub = threadIdx.x % 16;
  const bool live = col <= V;
  const bool vec = D % 4 == 0;
  const float q_scale = 1.0f / sqrtf((float)D);
  float* column = state + (int64_t)slots[run.x] * slot_stride + ((int64_t)h * (V + 1) + (live ? col : 0)) * D;
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
  for (int first = 0; first < run.z; first += MM_STEPS) {
    const int n = min(MM_STEPS, run.z - first);
    __syncthreads();  // the tokens before have been worked through
    for (int e = threadIdx.x; e < n * 2 * (DP / 4); e += 256) {
      const int which = e / (DP / 4), d = e % (DP / 4) * 4, i = which / 2;
      const T* row = proj + (int64_t)(run.y + first + i) * row_stride + ((which % 2) * H + h) * (int64_t)D;
      float x[4];
      load_row4(row, d, D, rows_vec, 0, x);
      if (which % 2) *reinterpret_cast<float4*>(s_k + i * DP + d) = make_float4(x[0], x[1], x[2], x[3]);
      else *reinterpret_cast<float4*>(s_q + i * DP + d) = make_float4(x[0] * q_scale, x[1] * q_scale, x[2] * q_scale, x[3] * q_scale);
    }
    float v[MM_STEPS], keep[MM_STEPS];
#pragma unroll
    for (int i = 0; i < MM_STEPS; ++i) {
      v[i] = keep[i] = 0.f;
      if (i < n && live) {
        const int64_t t = run.y + first + i;
        keep[i] = gates.keep[t * H + h];
        v[i] = gates.take[t * H + h] * (col < V ? to_f32(proj[t * row_stride + 2 * H * (int64_t)D + h * V + col]) : 1.f);
      }
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < MM_STEPS; ++i) {
      if (i >= n) break;
      float o = 0.f;
#pragma unroll
      for (int r = 0; r < R; ++r) {
        const float4 k4 = *reinterpret_cast<const float4*>(s_k + i * DP + 64 * r + 4 * sub);
        const float4 q4 = *reinterpret_cast<const float4*>(s_q + i * DP + 64 * r + 4 * sub);
        S[r][0] = fmaf(k4.x, v[i], keep[i] * S[r][0]); o = fmaf(S[r][0], q4.x, o);
        S[r][1] = fmaf(k4.y, v[i], keep[i] * S[r][1]); o = fmaf(S[r][1], q4.y, o);
        S[r][2] = fmaf(k4.z, v[i], keep[i] * S[r][2]); o = fmaf(S[r][2], q4.z, o);
        S[r][3] = fmaf(k4.w, v[i], keep[i] * S[r][3]); o = fmaf(S[r][3], q4.w, o);
      }
      o = sum16(o);
      if (live && sub == 0) {
        const int64_t at = (int64_t)(run.y + first + i) * H + h;
        if (col < V) out[at * V + col] = o;
        else nq[at] = o;
      }
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
// The logarithm of the product of the keeps after token j up to token t of one chunk, from their sums in two parts.
__device__ __forceinline__ float log_between(float hi_t, float lo_t, float hi_j, float lo_j) {
  return (hi_t - hi_j) + (lo_t - lo_j);
}

// chunks[c] = (table row of the sequence, first flat row, rows n <= CH, unused).  One workgroup (CH / 16 wavefronts) per
// (chunk, head, MM_VS value features): sums [chunk][H][V + 1][D], row V by the workgroup of the first features.
template <typename T, int DT, int CH>
__global__ __launch_bounds__(CH * 4) void memory_chunk_sums_kernel(const T* __restrict__ proj, int64_t row_stride,
                                                                   const int4* __restrict__ chunks, MemoryGates gates, int H,
                                                                   int D, int V, float* __restrict__ sums) {
  constexpr int NT = CH * 4, DS = DT * 16 + 4, VST = MM_VS + 4;
  __shared__ __attribute__((aligned(16))) float s_k[CH * DS];
  __shared__ __attribute__((aligned(16))) float s_v[CH * VST];
  __shared__ float s_w[CH];
  const int4 chunk = chunks[blockIdx.x];
  const int h = blockIdx.y, v0 = blockIdx.z * MM_VS;
  const int n = chunk.z;
  const bool aligned = row_stride % 4 == 0 && (uintptr_t)proj % 16 == 0;
  const bool kvec = aligned && D % 4 == 0, vvec = aligned && V % 4 == 0 && 2 * H * D % 4 == 0;
  if (threadIdx.x < CH) {
    const int j = threadIdx.x;
    float w = 0.f;
    if (j < n) {
      const int64_t at = (int64_t)(chunk.y + j) * H + h, end = (int64_t)(chunk.y + n - 1) * H + h;
      w = gates.take[at] * expf(log_between(gates.log_hi[end], gates.log_lo[end], gates.log_hi[at], gates.log_lo[at]));
    }
    s_w[j] = w;
  }
  __syncthreads();
  for (int e = threadIdx.x; e < CH * DT * 4; e += NT) {
    const int j = e / (DT * 4), d = e % (DT * 4) * 4;
    float x[4] = {0.f, 0.f, 0.f, 0.f};
    if (j < n) {
      load_row4(proj + (int64_t)(chunk.y + j) * row_stride + (H + h) * (int64_t)D, d, D, kvec, 0, x);
      const float w = s_w[j];
#pragma unroll
      for (int i = 0; i < 4; ++i) x[i] *= w;
    }
    *reinterpret_cast<float4*>(s_k + j * DS + d) = make_float4(x[0], x[1], x[2], x[3]);
  }
  for (int e = threadIdx.x; e < CH * (MM_VS / 4); e += NT) {
    const int j = e / (MM_VS / 4), v = e % (MM_VS / 4) * 4;
    float x[4] = {0.f, 0.f, 0.f, 0.f};
    if (j < n && v0 + v < V)
      load_row4(proj + (int64_t)(chunk.y + j) * row_stride + 2 * H * (int64_t)D + h * V, v0 + v, V, vvec, 0, x);
    *reinterpret_cast<float4*>(s_v + j * VST + v) = make_float4(x[0], x[1], x[2], x[3]);
  }
  __syncthreads();
  const int lane = threadIdx.x % PAE_WAVE, wave = threadIdx.x / PAE_WAVE, col = lane % 16, g4 = lane / 16;
  float* dst = sums + ((int64_t)blockIdx.x * H + h) * (V + 1) * D;
  for (int dt = wave; dt < DT; dt += CH / 16) {
    if (dt * 16 >= D) break;
    f32x4 acc[MM_VS / 16];
#pragma unroll
    for (int vt = 0; vt < MM_VS / 16; ++vt) acc[vt] = (f32x4){0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int s = 0; s < CH / 4; ++s) {
      const int j = 4 * s + g4;
      const float b = s_k[j * DS + dt * 16 + col];
#pragma unroll
      for (int vt = 0; vt < MM_VS / 16; ++vt)
        acc[vt] = __builtin_amdgcn_mfma_f32_16x16x4f32(s_v[j * VST + vt * 16 + col], b, acc[vt], 0, 0, 0);
    }
    const int d = dt * 16 + col;
    if (d < D) {
#pragma unroll
      for (int vt = 0; vt < MM_VS / 16; ++vt)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int v = v0 + vt * 16 + 4 * g4 + i;
          if (v < V) dst[(int64_t)v * D + d] = acc[vt][i];
        }
    }
  }
  if (blockIdx.z == 0)
    for (int d = threadIdx.x; d < D; d += NT) {
      float sum = 0.f;
      for (int j = 0; j < n; ++j) sum += s_k[j * DS + d];
      dst[(int64_t)V * D + d] = sum;
    }
}

// A thread per element of the state: sums become the states before every chunk, and the slot receives the state after
// the last.
template <int CH>
__global__ __launch_bounds__(256) void memory_chunk_scan_kernel(float* __restrict__ sums, const int4* __restrict__ chunks,
                                                                const int4* __restrict__ scans, const int* __restrict__ slots,
                                                                float* __restrict__ state, int64_t slot_stride,
                                                                const float* __restrict__ reach, int H, int64_t per_head,
                                                                int64_t total) {
  const int64_t e = (int64_t)blockIdx.x * 256 + threadIdx.x;
  if (e >= total) return;
  const int4 scan = scans[blockIdx.y];
  const float* keeps = reach + (int64_t)chunks[scan.y].y * H + e / per_head;  // of the run's first token and this head
  float* held = state + (int64_t)slots[scan.x] * slot_stride + e;
  float* at = sums + (int64_t)scan.y * total + e;
  float S = *held;
  constexpr int AHEAD = 8;
  for (int c0 = 0; c0 < scan.z; c0 += AHEAD) {
    float added[AHEAD], keep[AHEAD];
#pragma unroll
    for (int i = 0; i < AHEAD; ++i) {
      const int c = c0 + i;
      const bool there = c < scan.z;
      added[i] = there ? at[c * total] : 0.f;
      keep[i] = there ? keeps[((int64_t)c * CH + (c + 1 == scan.z ? scan.w : CH) - 1) * H] : 0.f;
    }
#pragma unroll
    for (int i = 0; i < AHEAD; ++i) {
      if (c0 + i >= scan.z) break;
      at[(c0 + i) * total] = S;
      S = fmaf(keep[i], S, added[i]);
    }
  }
  *held = S;
}

// One workgroup per (chunk, head, MM_VS value features); wavefront w has the queries 16 w .. 16 w + 15.  The scores are
// formed as K Q^T, whose accumulator (row = key 4 g4 + i, column = query) is the second product's B operand as it is.
template <typename T, int DT, int CH>
__global__ __launch_bounds__(CH * 4) void memory_chunk_out_kernel(const T* __restrict__ proj, int64_t row_stride,
                                                                  const int4* __restrict__ chunks, MemoryGates gates, int H,
                                                                  int D, int V, const float* __restrict__ before,
                                                                  float* __restrict__ out, float* __restrict__ nq) {
  constexpr int NT = CH * 4, DS = DT * 16 + 4, VST = MM_VS + 4;
  __shared__ __attribute__((aligned(16))) float s_k[CH * DS];
  __shared__ __attribute__((aligned(16))) float s_v[CH * VST];
  __shared__ float s_take[CH], s_hi[CH], s_lo[CH];
  const int4 chunk = chunks[blockIdx.x];
  const int h = blockIdx.y, v0 = blockIdx.z * MM_VS;
  const int n = chunk.z;
  const bool aligned = row_stride % 4 == 0 && (uintptr_t)proj % 16 == 0;
  const bool kvec = aligned && D % 4 == 0, vvec = aligned && V % 4 == 0 && 2 * H * D % 4 == 0;
  const int lane = threadIdx.x % PAE_WAVE, wave = threadIdx.x / PAE_WAVE, col = lane % 16, g4 = lane / 16;
  const int query = wave * 16 + col;  // this lane's query within the chunk
  const float q_scale = 1.0f / sqrtf((float)D);
  float q[DT][4];                     // features 16 s + 4 g4 + i of it
#pragma unroll
  for (int s = 0; s < DT; ++s) {
#pragma unroll
    for (int i = 0; i < 4; ++i) q[s][i] = 0.f;
    if (query < n) load_row4(proj + (int64_t)(chunk.y + query) * row_stride + h * (int64_t)D, 16 * s + 4 * g4, D, kvec, 0, q[s]);
#pragma unroll
    for (int i = 0; i < 4; ++i) q[s][i] *= q_scale;
  }
  for (int e = threadIdx.x; e < CH * DT * 4; e += NT) {
    const int j = e / (DT * 4), d = e % (DT * 4) * 4;
    float x[4] = {0.f, 0.f, 0.f, 0.f};
    if (j < n) load_row4(proj + (int64_t)(chunk.y + j) * row_stride + (H + h) * (int64_t)D, d, D, kvec, 0, x);
    *reinterpret_cast<float4*>(s_k + j * DS + d) = make_float4(x[0], x[1], x[2], x[3]);
  }
  for (int e = threadIdx.x; e < CH * (MM_VS / 4); e += NT) {
    const int j = e / (MM_VS / 4), v = e % (MM_VS / 4) * 4;
    float x[4] = {0.f, 0.f, 0.f, 0.f};
    if (j < n && v0 + v < V)
      load_row4(proj + (int64_t)(chunk.y + j) * row_stride + 2 * H * (int64_t)D + h * V, v0 + v, V, vvec, 0, x);
    *reinterpret_cast<float4*>(s_v + j * VST + v) = make_float4(x[0], x[1], x[2], x[3]);
  }
  if (threadIdx.x < CH) {
    const int64_t at = (int64_t)(chunk.y + min((int)threadIdx.x, n - 1)) * H + h;
    s_take[threadIdx.x] = gates.take[at];
    s_hi[threadIdx.x] = gates.log_hi[at];
    s_lo[threadIdx.x] = gates.log_lo[at];
  }
  __syncthreads();
  if (wave * 16 >= n) return;  // no barrier follows
  f32x4 acc[MM_VS / 16];
#pragma unroll
  for (int vt = 0; vt < MM_VS / 16; ++vt) acc[vt] = (f32x4){0.f, 0.f, 0.f, 0.f};
  // what the state before the chunk holds for these queries
  const float* S = before + ((int64_t)blockIdx.x * H + h) * (V + 1) * D;
  const bool svec = D % 4 == 0;
  const bool first_features = blockIdx.z == 0;  // this workgroup also reads out n
  float n_dot = 0.f;
#pragma unroll
  for (int s = 0; s < DT; ++s) {
    const int d = 16 * s + 4 * g4;
    if (16 * s >= D) break;
    float sv[MM_VS / 16][4];
#pragma unroll
    for (int vt = 0; vt < MM_VS / 16; ++vt) {
      const int v = v0 + vt * 16 + col;
      if (svec && v < V && d < D) {
        const float4 x = *reinterpret_cast<const float4*>(S + (int64_t)v * D + d);
        sv[vt][0] = x.x; sv[vt][1] = x.y; sv[vt][2] = x.z; sv[vt][3] = x.w;
      } else {
#pragma unroll
        for (int i = 0; i < 4; ++i) sv[vt][i] = v < V && d + i < D ? S[(int64_t)v * D + d + i] : 0.f;
      }
    }
    if (first_features) {
#pragma unroll
      for (int i = 0; i < 4; ++i)
        if (d + i < D) n_dot = fmaf(S[(int64_t)V * D + d + i], q[s][i], n_dot);
    }
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int vt = 0; vt < MM_VS / 16; ++vt)
        acc[vt] = __builtin_amdgcn_mfma_f32_16x16x4f32(sv[vt][i], q[s][i], acc[vt], 0, 0, 0);
  }
  const float hi = s_hi[query], lo = s_lo[query];  // (a query past the end has the last token's)
  const float reach = expf(hi);
  n_dot *= reach;
#pragma unroll
  for (int vt = 0; vt < MM_VS / 16; ++vt)
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
      const int j = jt * 16 + 4 * g4 + i;
      p[i] = j <= query ? p[i] * s_take[j] * expf(log_between(hi, lo, s_hi[j], s_lo[j])) : 0.f;
      n_dot += p[i];
    }
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
      for (int vt = 0; vt < MM_VS / 16; ++vt)
        acc[vt] = __builtin_amdgcn_mfma_f32_16x16x4f32(s_v[(jt * 16 + 4 * g4 + i) * VST + vt * 16 + col], p[i], acc[vt], 0, 0, 0);
  }
  n_dot += __shfl_xor(n_dot, 16, PAE_WAVE);
  n_dot += __shfl_xor(n_dot, 32, PAE_WAVE);
  if (query >= n) return;
  const int64_t at = (int64_t)(chunk.y + query) * H + h;
  if (first_features && g4 == 0) nq[at] = n_dot;
  float* dst = out + at * V;
#pragma unroll
  for (int vt = 0; vt < MM_VS / 16; ++vt) {
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

// ---------------------------------------------------------------------------------------------- division, norm, gate
// A wavefront per (token, head), four heads a workgroup; W features a lane at a time (2: all rows start on even features
// of rows aligned for pairs).
template <typename T, int W>
__global__ __launch_bounds__(256) void memory_finish_kernel(const float* __restrict__ o, const float* __restrict__ nq,
                                                            const float* __restrict__ floors, const T* __restrict__ gates,
                                                            int64_t gate_stride, const void* __restrict__ weight, int w_is_f32,
                                                            float eps, float floor_eps, int H, int V, T* __restrict__ out) {
  const int64_t t = blockIdx.x;
  const int h = blockIdx.y * 4 + threadIdx.x / PAE_WAVE, lane = threadIdx.x % PAE_WAVE;
  if (h >= H) return;
  const float* x = o + (t * H + h) * V;
  const float denom = fmaxf(fabsf(nq[t * H + h]), floors[t * H + h]) + floor_eps;
  float ss = 0.f;
  struct alignas(W * sizeof(float)) Floats { float v[W]; };
  struct alignas(W * sizeof(T)) Few { T v[W]; };
  for (int i = lane * W; i < V; i += PAE_WAVE * W) {
    const Floats a = *reinterpret_cast<const Floats*>(x + i);
#pragma unroll
    for (int e = 0; e < W; ++e) {
      const float y = a.v[e] / denom;
      ss = fmaf(y, y, ss);
    }
  }
  ss = wave_sum(ss);
  const float inv = 1.0f / sqrtf(ss / (float)V + eps);
  const T* gate = gates + t * gate_stride + h * V;
  for (int i = lane * W; i < V; i += PAE_WAVE * W) {
    const Floats a = *reinterpret_cast<const Floats*>(x + i);
    const Few z = *reinterpret_cast<const Few*>(gate + i);
    Few r;
#pragma unroll
    for (int e = 0; e < W; ++e) {
      const float g = 1.0f / (1.0f + expf(-to_f32(z.v[e])));
      r.v[e] = from_f32<T>(a.v[e] / denom * inv * load_param(weight, w_is_f32, h * V + i + e) * g);
    }
    *reinterpret_cast<Few*>(out + (t * H + h) * V + i) = r;
  }
}

// Tokens a chunk for key width D; 0: such heads take the serial kernel for runs of any length.
extern "C" int pae_matrix_memory_chunk(int D) { return D <= 128 ? 64 : (D <= 256 ? 32 : 0); }

struct MemoryStep {
  int64_t row_stride, gate_stride, state_slot_stride, max_slot_stride;
  const float* gate_logits;
  const void *x, *gate_w;
  int64_t ldx;
  const float* gate_b;
  int hidden;
  const int4 *serial, *chunks, *scans;
  int num_tokens, num_serial, num_chunks, num_scans;
  const int* slots;
  int H, D, V;
  float cap;
  float *state, *maximum;
  MemoryGates gates;
  float *sums, *o, *nq;
};

template <typename T>
static void memory_launch(const T* proj, const MemoryStep& a, hipStream_t stream) {
  const int H = a.H, D = a.D, V = a.V;
  if (a.num_serial > 0) {
    const int vec = 16 / (int)sizeof(T);
    const int wide = a.x && a.hidden % vec == 0 && a.ldx % vec == 0 && (uintptr_t)a.x % 16 == 0 && (uintptr_t)a.gate_w % 16 == 0;
    memory_gates_few_kernel<T><<<dim3(a.num_serial, H), 256, 0, stream>>>(a.gate_logits, (const T*)a.x, a.ldx, (const T*)a.gate_w,
                                                                          a.gate_b, a.hidden, wide, a.serial, a.slots, a.maximum,
                                                                          a.max_slot_stride, H, a.cap, a.gates);
    dim3 grid(a.num_serial, H, (V + 16) / 16);
#define MEMORY_SERIAL(R)                                                                                                \
  memory_serial_kernel<T, R><<<grid, 256, 0, stream>>>(proj, a.row_stride, a.serial, a.slots, a.state, a.state_slot_stride, \
                                                       a.gates, H, D, V, a.o, a.nq)
    if (D <= 64) MEMORY_SERIAL(1);
    else if (D <= 128) MEMORY_SERIAL(2);
    else if (D <= 256) MEMORY_SERIAL(4);
    else if (D <= 512) MEMORY_SERIAL(8);
    else MEMORY_SERIAL(16);
#undef MEMORY_SERIAL
  }
  if (a.num_chunks > 0) {
    dim3 grid(a.num_chunks, H, (V + MM_VS - 1) / MM_VS);
    const int64_t per_head = (int64_t)(V + 1) * D, total = H * per_head;
    dim3 scan_grid((unsigned)((total + 255) / 256), a.num_scans);
#define MEMORY_CHUNKS(DT, CH)                                                                                            \
  do {                                                                                                                   \
    memory_gates_scan_kernel<CH><<<dim3(H, a.num_scans), 1024, 0, stream>>>(a.gate_logits, a.chunks, a.scans, a.slots,   \
                                                                            a.maximum, a.max_slot_stride, H, a.cap, a.gates); \
    memory_chunk_sums_kernel<T, DT, CH><<<grid, CH * 4, 0, stream>>>(proj, a.row_stride, a.chunks, a.gates, H, D, V, a.sums); \
    memory_chunk_scan_kernel<CH><<<scan_grid, 256, 0, stream>>>(a.sums, a.chunks, a.scans, a.slots, a.state,             \
                                                                a.state_slot_stride, a.gates.reach, H, per_head, total); \
    memory_chunk_out_kernel<T, DT, CH><<<grid, CH * 4, 0, stream>>>(proj, a.row_stride, a.chunks, a.gates, H, D, V,      \
                                                                    a.sums, a.o, a.nq);                                  \
  } while (0)
    if (D <= 64) MEMORY_CHUNKS(4, 64);
    else if (D <= 128) MEMORY_CHUNKS(8, 64);
    else MEMORY_CHUNKS(16, 32);
#undef MEMORY_CHUNKS
  }
}

// `serial` int32 [num_serial][4], `chunks` [num_chunks][4], `scans` [num_scans][4] as the kernels above read them: between
// them they cover every row of the step once, a sequence in one of the lists only.  The gates' sums come as `gate_logits`
// [T][2 H] (input gates, then forget gates, biases included), or, where no run is in chunks, are formed here from the
// mixer's input `x` [T][hidden], `gate_w` [2 H][hidden] and `gate_b` [2 H].
extern "C" int pae_matrix_memory_step(int dtype, const void* proj, int64_t row_stride, const void* gate_in,
                                      int64_t gate_stride, const float* gate_logits, const void* x, int64_t ldx,
                                      const void* gate_w, const float* gate_b, int hidden, int num_tokens, const int* serial,
                                      int num_serial, const int* chunks, int num_chunks, const int* scans, int num_scans,
                                      const int* slots, int H, int D, int V, float gate_cap, float* state,
                                      int64_t state_slot_stride, float* maximum, int64_t max_slot_stride, const void* norm_w,
                                      int w_is_f32, float norm_eps, float floor_eps, float* work, void* out,
                                      hipStream_t stream) {
  PAE_REQUIRE(H > 0 && D > 0 && V > 0, "matrix memory: bad head sizes H=%d D=%d V=%d", H, D, V);
  PAE_REQUIRE(D <= 1024 && V <= 65535, "matrix memory: key width %d or value width %d exceeds the kernels' limits", D, V);
  PAE_REQUIRE(H <= 65535 && num_scans <= 65535, "matrix memory: %d heads, %d runs exceed the grid", H, num_scans);
  PAE_REQUIRE(row_stride >= 2 * (int64_t)H * D + (int64_t)H * V, "matrix memory: row stride %lld too small", (long long)row_stride);
  PAE_REQUIRE(gate_in && gate_stride >= (int64_t)H * V, "matrix memory: the gate's rows are missing or too narrow");
  PAE_REQUIRE(gate_cap > 0.f, "matrix memory: the gates' cap must be positive, got %g", (double)gate_cap);
  PAE_REQUIRE(gate_logits || (num_chunks == 0 && x && gate_w && gate_b && hidden > 0 && ldx >= hidden),
              "matrix memory: the gates' sums, or what they are formed from, are missing");
  PAE_REQUIRE(num_chunks == 0 || pae_matrix_memory_chunk(D) > 0, "matrix memory: key width %d has no chunks", D);
  PAE_REQUIRE((num_chunks == 0) == (num_scans == 0), "matrix memory: %d chunks with %d runs", num_chunks, num_scans);
  PAE_REQUIRE(dtype == PAE_F32 || dtype == PAE_BF16, "matrix memory: unknown dtype code %d", dtype);
  if (num_tokens <= 0) return 0;
  const int64_t TH = (int64_t)num_tokens * H;
  MemoryStep a{};
  a.row_stride = row_stride; a.gate_stride = gate_stride;
  a.state_slot_stride = state_slot_stride; a.max_slot_stride = max_slot_stride;
  a.gate_logits = gate_logits; a.x = x; a.ldx = ldx; a.gate_w = gate_w; a.gate_b = gate_b; a.hidden = hidden;
  a.serial = (const int4*)serial; a.chunks = (const int4*)chunks; a.scans = (const int4*)scans;
  a.num_tokens = num_tokens; a.num_serial = num_serial; a.num_chunks = num_chunks; a.num_scans = num_scans;
  a.slots = slots; a.H = H; a.D = D; a.V = V; a.cap = gate_cap; a.state = state; a.maximum = maximum;
  // work: o [T][H][V], sums [num_chunks][H][V + 1][D], each from a 16-byte boundary on; then seven of [T][H]
  a.o = work;
  a.sums = a.o + (TH * V + 3) / 4 * 4;
  float* rest = a.sums + ((int64_t)num_chunks * H * (V + 1) * D + 3) / 4 * 4;
  a.nq = rest;
  a.gates = MemoryGates{rest + TH, rest + 2 * TH, rest + 3 * TH, rest + 4 * TH, rest + 5 * TH, rest + 6 * TH};
  dim3 token_heads(num_tokens, (H + 3) / 4);
  const int size = dtype == PAE_F32 ? 4 : 2;
  const bool pairs = V % 2 == 0 && gate_stride % 2 == 0 && (uintptr_t)gate_in % (2 * size) == 0 && (uintptr_t)out % (2 * size) == 0;
#define MEMORY_FINISH(T, W)                                                                                              \
  memory_finish_kernel<T, W><<<token_heads, 256, 0, stream>>>(a.o, a.nq, a.gates.floors, (const T*)gate_in, gate_stride,  \
                                                              norm_w, w_is_f32, norm_eps, floor_eps, H, V, (T*)out)
  if (dtype == PAE_F32) {
    memory_launch((const float*)proj, a, stream);
    if (pairs) MEMORY_FINISH(float, 2);
    else MEMORY_FINISH(float, 1);
  } else {
    memory_launch((const bf16_t*)proj, a, stream);
    if (pairs) MEMORY_FINISH(bf16_t, 2);
    else MEMORY_FINISH(bf16_t, 1);
  }
#undef MEMORY_FINISH
  return pae_check_launch("matrix_memory_step");
}

// floats of `work` that pae_matrix_memory_step needs
extern "C" int64_t pae_matrix_memory_work_floats(int num_tokens, int num_chunks, int H, int D, int V) {
  const int64_t TH = (int64_t)num_tokens * H;
  return (TH * V + 3) / 4 * 4 + ((int64_t)num_chunks * H * (V + 1) * D + 3) / 4 * 4 + 7 * TH;
}
