// A matrix memory per head whose rows decay one by one and from which, token by token, a part of what the unit key reads is
// removed along another direction:
//   u = k / sqrt(sum(k^2) + 1e-6),   w = exp(-exp(-1/2) sigmoid(raw_w + w0)),   a = sigmoid(raw_a + bias_a)     per head and row
//   S_t = diag(w) S_(t-1) - (a u) (u^T S_(t-1)) + k v^T   (both terms read the old state),   o_t = S_t^T r,
// and behind it, per head, o / sqrt(mean(o^2) + eps) * weight * sigmoid(gate).
//
// A batch is token-major without padding: sequence s owns rows cu_seqlens[s] .. cu_seqlens[s + 1] - 1, its state sits in
// slot state_slots[s] as [heads][d][d] floats (row n, column p), and seq_starts[s] == 0 says that it starts now, from a zero
// state, whatever the slot held.  All arithmetic is float; T is the storage type of the rows.
#include "common.h"

using namespace pllm;

struct DeltaArgs {
  // rows [T, heads * d] each, head by head, with a common row stride: columns r_at, k_at, v_at, a_at, g_at of `rows`
  const void* rows; long stride;
  int r_at, k_at, v_at, a_at, g_at;
  const float* raw_w; long w_stride;       // [T, heads * d]
  const float* w0; const float* bias_a;    // [heads * d]
  const float* weight; float eps;          // of the norm behind the memory: [heads * d]
  float* state; long slot_stride;
  const int* state_slots; const int* seq_starts; const int* cu_seqlens;
  void* out;                               // [T, heads * d]
  int heads, d;
};

__device__ __forceinline__ float sigmoid_f32(float z) { return 1.f / (1.f + expf(-z)); }
constexpr float kDecayRate = 0.60653065971263342f;      // exp(-1/2)
constexpr float kUnitEps = 1e-6f;

// Token by token: one workgroup per (head, sequence), lane = column of S in each of CB blocks of 64 columns, wavefront w holds
// rows w * 16 .. w * 16 + 15 in registers.  A lane below 16 makes its row's decay, removal rate and unit key; they are read
// out lane by lane.  With q = S_(t-1)^T u the output is sum_n r_n w_n S_n - (sum_n r_n a_n u_n) q + (sum_n r_n k_n) v, so the
// wavefronts exchange both sums of a token at once: one barrier a token.  The norm and the gate follow in the same kernel.
constexpr int kDeltaRows = 16;

template <typename T, int CB, int MAX_THREADS>
__global__ __launch_bounds__(MAX_THREADS) void delta_rule_kernel(DeltaArgs a) {
  constexpr int MAX_WAVES = MAX_THREADS / 64;
  __shared__ float part_q[2][MAX_WAVES][CB * 64], part_o[2][MAX_WAVES][CB * 64], part_s[2][MAX_WAVES][2];
  const int lane = threadIdx.x & 63, wv = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), waves = blockDim.x >> 6;
  const int head = blockIdx.x, seq = blockIdx.y, d = a.d;
  const int q_begin = a.cu_seqlens[seq], q_len = a.cu_seqlens[seq + 1] - q_begin;
  if (q_len <= 0) return;                                      // the whole workgroup: no barrier is left behind
  float* st = a.state + (size_t)a.state_slots[seq] * a.slot_stride + (size_t)head * d * d;
  const bool carried = a.seq_starts[seq] > 0;
  const int n0 = wv * kDeltaRows;
  float S[CB][kDeltaRows];
#pragma unroll
  for (int b = 0; b < CB; ++b)
#pragma unroll
    for (int i = 0; i < kDeltaRows; ++i)
      S[b][i] = (carried && n0 + i < d && b * 64 + lane < d) ? st[(size_t)(n0 + i) * d + b * 64 + lane] : 0.f;
  const T* rows = reinterpret_cast<const T*>(a.rows) + (size_t)q_begin * a.stride + (size_t)head * d;
  const float* raw_w = a.raw_w + (size_t)q_begin * a.w_stride + (size_t)head * d;
  T* out = reinterpret_cast<T*>(a.out) + (size_t)q_begin * a.heads * d + (size_t)head * d;
  const bool mine = lane < kDeltaRows && n0 + lane < d;        // this lane makes row n0 + lane
  const int nn = mine ? n0 + lane : 0;
  const float w0 = mine ? a.w0[(size_t)head * d + nn] : 0.f, bias_a = mine ? a.bias_a[(size_t)head * d + nn] : 0.f;
  float weight[CB];
#pragma unroll
  for (int b = 0; b < CB; ++b) weight[b] = b * 64 + lane < d ? a.weight[(size_t)head * d + b * 64 + lane] : 0.f;
  struct Fetched { float r, k, w, a, v[CB], key[CB], g[CB]; };
  auto fetch = [&](int t) {
    Fetched f;
    const T* row = rows + (size_t)t * a.stride;
    f.r = mine ? to_f32(row[a.r_at + nn]) : 0.f;
    f.k = mine ? to_f32(row[a.k_at + nn]) : 0.f;
    f.a = mine ? to_f32(row[a.a_at + nn]) : 0.f;
    f.w = mine ? raw_w[(size_t)t * a.w_stride + nn] : 0.f;
#pragma unroll
    for (int b = 0; b < CB; ++b) {
      const bool in = b * 64 + lane < d;
      const int p = in ? b * 64 + lane : 0;
      f.v[b] = in ? to_f32(row[a.v_at + p]) : 0.f;
      f.key[b] = in ? to_f32(row[a.k_at + p]) : 0.f;
      f.g[b] = in ? to_f32(row[a.g_at + p]) : 0.f;
    }
    return f;
  };
  Fetched next = fetch(0);
  for (int t = 0; t < q_len; ++t) {
    const Fetched f = next;
    if (t + 1 < q_len) next = fetch(t + 1);
    float ksq = 0.f;
#pragma unroll
    for (int b = 0; b < CB; ++b) ksq = fmaf(f.key[b], f.key[b], ksq);
    const float inv_k = 1.f / sqrtf(wave_sum(ksq) + kUnitEps);
    const float u_l = f.k * inv_k;
    const float w_l = mine ? expf(-kDecayRate * sigmoid_f32(f.w + w0)) : 0.f;
    const float b_l = mine ? sigmoid_f32(f.a + bias_a) * u_l : 0.f;
    const float rw_l = f.r * w_l;
    const float rb = wave_sum(f.r * b_l), rk = wave_sum(f.r * f.k);
    float q[CB], o[CB];
#pragma unroll
    for (int b = 0; b < CB; ++b) q[b] = o[b] = 0.f;
#pragma unroll
    for (int i = 0; i < kDeltaRows; ++i) {
      const float uu = row_lane(u_l, i), rr = row_lane(rw_l, i);
#pragma unroll
      for (int b = 0; b < CB; ++b) {
        q[b] = fmaf(uu, S[b][i], q[b]);
        o[b] = fmaf(rr, S[b][i], o[b]);
      }
    }
    const int buf = t & 1;
    float rb_all = rb, rk_all = rk;
    if (waves > 1) {
#pragma unroll
      for (int b = 0; b < CB; ++b) {
        part_q[buf][wv][b * 64 + lane] = q[b];
        part_o[buf][wv][b * 64 + lane] = o[b];
      }
      if (lane == 0) {
        part_s[buf][wv][0] = rb;
        part_s[buf][wv][1] = rk;
      }
      __syncthreads();
      rb_all = rk_all = 0.f;
#pragma unroll
      for (int b = 0; b < CB; ++b) q[b] = o[b] = 0.f;
      for (int w = 0; w < waves; ++w) {
        rb_all += part_s[buf][w][0];
        rk_all += part_s[buf][w][1];
#pragma unroll
        for (int b = 0; b < CB; ++b) {
          q[b] += part_q[buf][w][b * 64 + lane];
          o[b] += part_o[buf][w][b * 64 + lane];
        }
      }
    }
#pragma unroll
    for (int i = 0; i < kDeltaRows; ++i) {
      const float ww = row_lane(w_l, i), bb = row_lane(b_l, i), kk = row_lane(f.k, i);
#pragma unroll
      for (int b = 0; b < CB; ++b) S[b][i] = fmaf(kk, f.v[b], fmaf(-bb, q[b], ww * S[b][i]));
    }
    if (wv == t % waves) {                                      // one wavefront in turn finishes the token
      float sq = 0.f;
#pragma unroll
      for (int b = 0; b < CB; ++b) {
        o[b] = fmaf(rk_all, f.v[b], fmaf(-rb_all, q[b], o[b]));
        sq = fmaf(o[b], o[b], sq);                              // (columns past the head's last hold zeros)
      }
      const float inv = 1.f / sqrtf(wave_sum(sq) / (float)d + a.eps);
#pragma unroll
      for (int b = 0; b < CB; ++b)
        if (b * 64 + lane < d) out[(size_t)t * a.heads * d + b * 64 + lane] = from_f32<T>(o[b] * inv * weight[b] * sigmoid_f32(f.g[b]));
    }
  }
#pragma unroll
  for (int b = 0; b < CB; ++b)
#pragma unroll
    for (int i = 0; i < kDeltaRows; ++i)
      if (n0 + i < d && b * 64 + lane < d) st[(size_t)(n0 + i) * d + b * 64 + lane] = S[b][i];
}

template <typename T>
static void launch_delta(const DeltaArgs& a, int num_seqs, hipStream_t stream) {
  dim3 grid(a.heads, num_seqs), block(64 * ((a.d + kDeltaRows - 1) / kDeltaRows));
  if (a.d <= 64) hipLaunchKernelGGL((delta_rule_kernel<T, 1, 256>), grid, block, 0, stream, a);
  else if (a.d <= 128) hipLaunchKernelGGL((delta_rule_kernel<T, 2, 512>), grid, block, 0, stream, a);
  else hipLaunchKernelGGL((delta_rule_kernel<T, 4, 1024>), grid, block, 0, stream, a);
}

PLLM_API int pllm_delta_rule(int dtype, const void* rows, long stride, int r_at, int k_at, int v_at, int a_at, int g_at, const float* raw_w,
                             long w_stride, const float* w0, const float* bias_a, const float* weight, float eps, float* state,
                             long slot_stride, const int* state_slots, const int* seq_starts, const int* cu_seqlens, void* out, int num_seqs,
                             int heads, int d, hipStream_t stream) {
  if (num_seqs <= 0) return 0;
  if (heads <= 0 || d <= 0 || d > 256 || num_seqs > 65535) return -2;
  DeltaArgs a{rows, stride, r_at, k_at, v_at, a_at, g_at, raw_w, w_stride, w0, bias_a, weight, eps, state, slot_stride,
              state_slots, seq_starts, cu_seqlens, out, heads, d};
  if (dtype == PLLM_F32) launch_delta<float>(a, num_seqs, stream);
  else launch_delta<bf16>(a, num_seqs, stream);
  PLLM_RETURN_LAST_ERROR();
}
