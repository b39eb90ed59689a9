// Selective scan: a recurrence with a state of N floats per channel whose decays depend on the token and the channel,
//   s_c <- e^(step_c A_c) * s_c + (step_c x_c) B  for the N states s_c of channel c,   y_c = <s_c, C> + D_c x_c,
// and the gate behind it, out = y silu(z).  The step sizes arrive raw: step = softplus(raw + bias).
//
// A batch is token-major without padding: sequence s owns rows cu_seqlens[s] .. cu_seqlens[s + 1] - 1, its state sits in
// slot state_slots[s] as [N][channels] floats, and seq_starts[s] == 0 says that it starts now, from a zero state, whatever
// the slot held.  All arithmetic is float; T is the storage type of x, z and the output rows.
//
// One lane per channel with its states in registers.  B and C of a token are the same numbers for every channel, so a
// wavefront reads them through the scalar path (rows [T, 2 N] of type T, in the passes over chunks float: there taking pairs of
// bfloat16 elements apart would cost more than it saves).  N is 8, 16 or a multiple of 32: a caller with another
// size pads A, B and C with zeros, and the padded states stay zero.  States of more than 32 elements are cut over the
// workgroup's wavefronts, whose partial outputs meet in LDS.  A is held as A log2(e), so that a decay is one multiply and one
// hardware exponential.
#include "common.h"

using namespace pllm;

struct ScanArgs {
  const void* x; long x_stride;          // [T, channels]
  const float* raw;                      // raw step sizes [T, channels]
  float* dt;                             // chunks: softplus(raw + bias) [T, channels], which the first pass leaves for the third
  const float* dt_bias;                  // [channels]
  const float* a2;                       // [N][channels]: A log2(e)
  const float* skip;                     // [channels]
  const void* z; long z_stride;          // [T, channels]
  float* state; long slot_stride;
  const int* state_slots; const int* seq_starts; const int* cu_seqlens;
  void* out;                             // [T, channels]
  int channels, N, num_seqs;
  int chunk;                             // tokens per chunk (0: whole sequences)
  float* ws_state;                       // [chunks][N][channels]
  float* ws_steps;                       // [chunks][channels]: the sum of a chunk's step sizes
};

// log(1 + e^z) without losing small results: u = 1 + e^-|z| is rounded, and log(u) e / (u - 1) undoes what that lost.
__device__ __forceinline__ float softplus_f32(float z) {
  const float e = expf(-fabsf(z));
  const float u = 1.f + e;
  const float d = u - 1.f;
  const float l = d > 0.f ? logf(u) * (e / d) : e;
  return fmaxf(z, 0.f) + l;
}

// Element i of a row that the whole wavefront reads: bfloat16 elements come in pairs (the scalar path has no loads of 16 bits).
__device__ __forceinline__ float uniform_element(const float* row, int i) { return row[i]; }
__device__ __forceinline__ float uniform_element(const bf16* row, int i) {
  const uint32_t pair = reinterpret_cast<const uint32_t*>(row)[i >> 1];
  return __uint_as_float((i & 1) ? pair & 0xffff0000u : pair << 16);
}

enum { kScanWhole = 0, kScanState = 1, kScanOut = 2 };
constexpr int kScanAhead = 4;            // tokens whose rows are asked for at once

__device__ __forceinline__ bool scan_chunk_of(const int* __restrict__ cu, int num_seqs, int chunk, int j, int& seq, int& local) {
  int base = 0;
  for (int s = 0; s < num_seqs; ++s) {
    const int c = (cu[s + 1] - cu[s] + chunk - 1) / chunk;
    if (j < base + c) { seq = s; local = j - base; return true; }
    base += c;
  }
  return false;
}

// kScanWhole: a sequence's tokens of this step from the slot's state to the slot's state.  kScanState: a chunk's own
// contribution from a zero state, walked from its last token to its first (the decays behind a token are then one
// exponential of A times the step sizes summed so far), and the softplus of its step sizes.  kScanOut: a chunk's tokens
// from the state the sequence had when the chunk began.
template <typename T, typename TB, int NR, int MAX_THREADS, int MODE>
__global__ __launch_bounds__(MAX_THREADS) void selective_scan_kernel(ScanArgs a, const TB* __restrict__ bc, long bc_stride) {
  __shared__ float part[2][MAX_THREADS / 64][64];
  const int lane = threadIdx.x & 63, wv = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), waves = blockDim.x >> 6;
  int seq = blockIdx.y, local = 0;
  if (MODE != kScanWhole && !scan_chunk_of(a.cu_seqlens, a.num_seqs, a.chunk, blockIdx.y, seq, local)) return;
  const int q_begin = a.cu_seqlens[seq], q_len = a.cu_seqlens[seq + 1] - q_begin;
  if (q_len <= 0) return;
  const int t_first = MODE == kScanWhole ? 0 : local * a.chunk;
  const int t_last = MODE == kScanWhole ? q_len : min(t_first + a.chunk, q_len);
  const int c = blockIdx.x * 64 + lane;
  const bool ok = c < a.channels;
  const int cc = ok ? c : a.channels - 1;                     // (a lane past the last channel repeats it and stores nothing)
  const int n0 = wv * NR;
  const size_t C = a.channels;
  float* st = MODE == kScanWhole ? a.state + (size_t)a.state_slots[seq] * a.slot_stride : a.ws_state + (size_t)blockIdx.y * a.N * C;
  const bool from_state = MODE == kScanOut || (MODE == kScanWhole && a.seq_starts[seq] > 0);
  float S[NR], A[NR];
#pragma unroll
  for (int i = 0; i < NR; ++i) {
    A[i] = a.a2[(size_t)(n0 + i) * C + cc];
    S[i] = from_state ? st[(size_t)(n0 + i) * C + cc] : 0.f;
  }
  const float bias = a.dt_bias[cc], skip = a.skip[cc];
  const T* xp = reinterpret_cast<const T*>(a.x) + (size_t)q_begin * a.x_stride + cc;
  const T* zp = reinterpret_cast<const T*>(a.z) + (size_t)q_begin * a.z_stride + cc;
  const float* rp = (MODE == kScanOut ? a.dt : a.raw) + (size_t)q_begin * C + cc;
  float* dp = a.dt + (size_t)q_begin * C + cc;
  T* op = reinterpret_cast<T*>(a.out) + (size_t)q_begin * C + cc;
  float behind = 0.f;                                         // kScanState: the step sizes of the tokens behind, summed
  for (int tb = t_first; tb < t_last; tb += kScanAhead) {
    T xv[kScanAhead], zv[kScanAhead];
    float rv[kScanAhead];
#pragma unroll
    for (int u = 0; u < kScanAhead; ++u) {
      const int n = min(tb + u, t_last - 1);
      const int t = MODE == kScanState ? t_last - 1 - (n - t_first) : n;
      xv[u] = xp[(size_t)t * a.x_stride];
      rv[u] = rp[(size_t)t * C];
      if (MODE != kScanState) zv[u] = zp[(size_t)t * a.z_stride];
    }
#pragma unroll
    for (int u = 0; u < kScanAhead; ++u) {
      if (tb + u >= t_last) break;
      const int t = MODE == kScanState ? t_last - 1 - (tb + u - t_first) : tb + u;
      const float x = to_f32(xv[u]);
      const TB* row = bc + (size_t)(q_begin + t) * bc_stride;           // B, then C
      float dt = rv[u];
      if (MODE != kScanOut) dt = softplus_f32(dt + bias);     // (kScanOut: the first pass has left it)
      const float dx = dt * x;
      if (MODE == kScanState) {
        if (ok && wv == 0) dp[(size_t)t * C] = dt;
#pragma unroll
        for (int i = 0; i < NR; ++i) S[i] = fmaf(__builtin_amdgcn_exp2f(A[i] * behind), dx * uniform_element(row, n0 + i), S[i]);
        behind += dt;
        continue;
      }
      float y[2] = {0.f, 0.f};
#pragma unroll
      for (int i = 0; i < NR; ++i) {
        S[i] = fmaf(__builtin_amdgcn_exp2f(A[i] * dt), S[i], dx * uniform_element(row, n0 + i));
        y[i & 1] = fmaf(S[i], uniform_element(row, a.N + n0 + i), y[i & 1]);
      }
      float total = y[0] + y[1];
      if (waves > 1) {
        part[t & 1][wv][lane] = total;
        __syncthreads();
        total = part[t & 1][0][lane];
        for (int w = 1; w < waves; ++w) total += part[t & 1][w][lane];
      }
      if (ok && wv == 0) {
        const float z = to_f32(zv[u]);
        op[(size_t)t * C] = from_f32<T>(fmaf(skip, x, total) * (z / (1.f + expf(-z))));
      }
    }
  }
  if (MODE == kScanOut || !ok) return;
#pragma unroll
  for (int i = 0; i < NR; ++i) st[(size_t)(n0 + i) * C + c] = S[i];
  if (MODE == kScanState && wv == 0) a.ws_steps[(size_t)blockIdx.y * C + c] = behind;
}

// Between the two passes, per sequence and state element, chunk after chunk: ws <- the state before the chunk,
// S <- exp(A times the chunk's step sizes) S + the chunk's own contribution; the last state goes to the slot.
__global__ __launch_bounds__(256) void selective_scan_carry_kernel(ScanArgs a) {
  const size_t C = a.channels, per_seq = (size_t)a.N * C;
  const size_t idx = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
  const int seq = blockIdx.y;
  if (idx >= per_seq) return;
  const int q_len = a.cu_seqlens[seq + 1] - a.cu_seqlens[seq];
  if (q_len <= 0) return;
  int base = 0;
  for (int s = 0; s < seq; ++s) base += (a.cu_seqlens[s + 1] - a.cu_seqlens[s] + a.chunk - 1) / a.chunk;
  const int chunks = (q_len + a.chunk - 1) / a.chunk;
  const size_t c = idx % C;
  const float a2 = a.a2[idx];
  float* slot = a.state + (size_t)a.state_slots[seq] * a.slot_stride + idx;
  float* w = a.ws_state + (size_t)base * per_seq + idx;
  const float* steps = a.ws_steps + (size_t)base * C + c;
  float S = a.seq_starts[seq] > 0 ? *slot : 0.f;
  constexpr int kAhead = 8;                                   // chunks whose contributions are asked for at once
  for (int c0 = 0; c0 < chunks; c0 += kAhead) {
    float loc[kAhead], sum[kAhead];
#pragma unroll
    for (int u = 0; u < kAhead; ++u) {
      const int j = min(c0 + u, chunks - 1);
      loc[u] = w[(size_t)j * per_seq];
      sum[u] = steps[(size_t)j * C];
    }
#pragma unroll
    for (int u = 0; u < kAhead; ++u) {
      if (c0 + u >= chunks) break;
      w[(size_t)(c0 + u) * per_seq] = S;
      S = fmaf(__builtin_amdgcn_exp2f(a2 * sum[u]), S, loc[u]);
    }
  }
  *slot = S;
}

template <typename T, typename TB, int MODE>
static void launch_scan(const ScanArgs& a, const void* bc, long bc_stride, int rows, hipStream_t stream) {
  const int waves = (a.N + 31) / 32;
  dim3 grid((a.channels + 63) / 64, rows), block(64 * waves);
#define PLLM_SCAN(NR, MAX_THREADS) hipLaunchKernelGGL((selective_scan_kernel<T, TB, NR, MAX_THREADS, MODE>), grid, block, 0, stream, a, (const TB*)bc, bc_stride)
  if (a.N == 8) PLLM_SCAN(8, 256);
  else if (a.N == 16) PLLM_SCAN(16, 256);
  else if (waves <= 4) PLLM_SCAN(32, 256);
  else PLLM_SCAN(32, 1024);
#undef PLLM_SCAN
}

// bc: [T, 2 N] of type dtype, or (chunk > 0) float.  chunk == 0: every sequence token by token.  chunk > 0: three passes over chunks of that many tokens; ws_state holds
// max_chunks * N * channels floats and ws_steps max_chunks * channels, max_chunks >= sum over the sequences of
// ceil(q_len / chunk).
PLLM_API int pllm_selective_scan(int dtype, const void* x, long x_stride, const float* raw, float* dt, const float* dt_bias, const void* bc, long bc_stride,
                                 const float* a2, const float* skip, const void* z, long z_stride, float* state, long slot_stride,
                                 const int* state_slots, const int* seq_starts, const int* cu_seqlens, void* out, int num_seqs, int channels,
                                 int N, int chunk, int max_chunks, float* ws_state, float* ws_steps, hipStream_t stream) {
  if (num_seqs <= 0) return 0;
  if (channels <= 0 || (N != 8 && N != 16 && (N <= 0 || N % 32)) || N > 512 || num_seqs > 65535 || chunk < 0) return -2;
  if (chunk > 0 && (max_chunks <= 0 || max_chunks > 65535 || !ws_state || !ws_steps || !dt)) return -2;
  ScanArgs a{x, x_stride, raw, dt, dt_bias, a2, skip, z, z_stride, state, slot_stride, state_slots, seq_starts, cu_seqlens, out,
             channels, N, num_seqs, chunk, ws_state, ws_steps};
  if (chunk == 0) {
    if (dtype == PLLM_F32) launch_scan<float, float, kScanWhole>(a, bc, bc_stride, num_seqs, stream);
    else launch_scan<bf16, bf16, kScanWhole>(a, bc, bc_stride, num_seqs, stream);
    PLLM_RETURN_LAST_ERROR();
  }
  const size_t per_seq = (size_t)N * channels;
  if (dtype == PLLM_F32) launch_scan<float, float, kScanState>(a, bc, bc_stride, max_chunks, stream);
  else launch_scan<bf16, float, kScanState>(a, bc, bc_stride, max_chunks, stream);
  hipLaunchKernelGGL(selective_scan_carry_kernel, dim3((unsigned)((per_seq + 255) / 256), num_seqs), dim3(256), 0, stream, a);
  if (dtype == PLLM_F32) launch_scan<float, float, kScanOut>(a, bc, bc_stride, max_chunks, stream);
  else launch_scan<bf16, float, kScanOut>(a, bc, bc_stride, max_chunks, stream);
  PLLM_RETURN_LAST_ERROR();
}
