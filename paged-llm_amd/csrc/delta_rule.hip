// A matrix memory per head whose rows decay one by one and from which, token by token, a part of what the unit key reads is
// removed along another direction:
//   u = k / sqrt(sum(k^2) + 1e-6),   w = exp(-exp(-1/2) sigmoid(raw_w + w0)),   a = sigmoid(raw_a + bias_a)     per head and row
//   z = S^T u  (S as the token finds it),   S <- w . S - (a . u) z^T + k v^T  (w . S: row by row),   o = S^T r,
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

template <typename T, int CB, int AHEAD, int MAX_THREADS>
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
  // AHEAD tokens' rows are asked for while the AHEAD tokens before are worked off
  Fetched next[AHEAD];
#pragma unroll
  for (int e = 0; e < AHEAD; ++e)
    if (e < q_len) next[e] = fetch(e);
  for (int tb = 0; tb < q_len; tb += AHEAD) {
   Fetched now[AHEAD];
#pragma unroll
   for (int e = 0; e < AHEAD; ++e) {
     now[e] = next[e];
     if (tb + AHEAD + e < q_len) next[e] = fetch(tb + AHEAD + e);
   }
#pragma unroll
   for (int e = 0; e < AHEAD; ++e) {
    const int t = tb + e;
    if (t >= q_len) break;
    const Fetched f = now[e];
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
  if (a.d <= 64) hipLaunchKernelGGL((delta_rule_kernel<T, 1, 4, 256>), grid, block, 0, stream, a);
  else if (a.d <= 128) hipLaunchKernelGGL((delta_rule_kernel<T, 2, 2, 512>), grid, block, 0, stream, a);
  else hipLaunchKernelGGL((delta_rule_kernel<T, 4, 1, 1024>), grid, block, 0, stream, a);
}

// (pllm_delta_rule: token by token, any length.)
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

// ---------------------------------------------------------------------------------------------
// Long portions.  A chunk of C = 32 tokens is worked off as matrices.  With G_t the product of the decays of the chunk's tokens
// up to t (a number per row of S), S the state in front of the chunk and z_t = S_(t-1)^T u_t what token t reads,
//   S_t = G_t S + sum_{j <= t} (G_t / G_j) (k_j v_j^T - b_j z_j^T),   b = a u,
//   (I + L_b) Z = U S + L_k V,                     U_t = G_(t-1) u_t,  L_x[t, j] = U_t . (x_j / G_j) for j < t
//   O = R S + A_k V - A_b Z,                       R_t = G_t r_t,      A_x[t, j] = R_t . (x_j / G_j) for j <= t
//   S_C = G_C S + sum_j (G_C / G_j) (k_j v_j^T - b_j z_j^T).
// (A decay lies between exp(-exp(-1/2)) and 1, so 1 / G_j stays below 3e8 and every product G_t / G_j that is used is at most 1.)
// delta_chunk_kernel makes, for all chunks side by side, what does not depend on the state: with X = (I + L_b)^-1
//   U' = X U,  V' = X L_k V,  R' = R - A_b U',  O' = A_k V - A_b V',  K' = G_C / G_j k_j,  B' = -G_C / G_j b_j,
// and delta_carry_kernel walks a sequence's chunks with a block of 16 columns of S:  Z = U' S + V',  O = R' S + O',
// S <- G_C S + K'^T V + B'^T Z.  All products run on the matrix cores in float (v_mfma_f32_16x16x4_f32).
//
// What the first leaves for the second lies in the operands' order: a fragment of 256 floats is 16 rows x 16 elements of
// k, lane (g, m) = (lane >> 4, lane & 15) holding row m, elements 4 g .. 4 g + 3, which feed four instructions (the same
// assignment of k on both sides); a result's lane (g, c) holds rows 4 g .. 4 g + 3 of column c and is such a fragment of
// the next product as it stands.
constexpr int kDeltaChunk = 32;
constexpr int kChunkMaxDim = 128;        // heads up to this size; larger ones go token by token
typedef __attribute__((ext_vector_type(4))) float delta_floatx4;

struct DeltaChunks {
  float* ur;       // [chunk][head][4][DT] fragments: rows of U' (two tiles of 16 tokens), rows of R'
  float* vo;       // [chunk][head][4][DT] fragments in the result's order: V', O' by tiles of tokens and of columns
  float* kb;       // [chunk][head][DT][4] fragments: K'^T, B'^T (rows of S by tiles; the chunk's tokens in two halves each)
  float* vf;       // [chunk][head][DT][2] fragments: V by tiles of columns, tokens in two halves
  float* gamma;    // [chunk][head][16 DT]: G_C
  float* y;        // [T][heads * d]: O
  int num_seqs, max_chunks, DT;
};

__device__ __forceinline__ bool delta_chunk_of(const int* __restrict__ cu, int num_seqs, int j, int& seq, int& local) {
  int base = 0;
  for (int s = 0; s < num_seqs; ++s) {
    const int c = (cu[s + 1] - cu[s] + kDeltaChunk - 1) / kDeltaChunk;
    if (j < base + c) { seq = s; local = j - base; return true; }
    base += c;
  }
  return false;
}

__device__ __forceinline__ delta_floatx4 lds4(const float* p) { return *reinterpret_cast<const delta_floatx4*>(p); }
__device__ __forceinline__ delta_floatx4 mfma4(const delta_floatx4 a, const delta_floatx4 b, delta_floatx4 acc) {
#pragma unroll
  for (int i = 0; i < 4; ++i) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a[i], b[i], acc, 0, 0, 0);
  return acc;
}

__device__ __forceinline__ void load8(const float* p, float* v, bool on) {
  const float4 lo = on ? reinterpret_cast<const float4*>(p)[0] : make_float4(0.f, 0.f, 0.f, 0.f);
  const float4 hi = on ? reinterpret_cast<const float4*>(p)[1] : make_float4(0.f, 0.f, 0.f, 0.f);
  v[0] = lo.x; v[1] = lo.y; v[2] = lo.z; v[3] = lo.w; v[4] = hi.x; v[5] = hi.y; v[6] = hi.z; v[7] = hi.w;
}
__device__ __forceinline__ void load8(const bf16* p, float* v, bool on) {
  const uint4 q = on ? *reinterpret_cast<const uint4*>(p) : make_uint4(0, 0, 0, 0);
  const uint32_t w[4] = {q.x, q.y, q.z, q.w};
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    v[2 * i] = __uint_as_float(w[i] << 16);
    v[2 * i + 1] = __uint_as_float(w[i] & 0xffff0000u);
  }
}
__device__ __forceinline__ void store8(float* p, const float* v) {
  reinterpret_cast<float4*>(p)[0] = make_float4(v[0], v[1], v[2], v[3]);
  reinterpret_cast<float4*>(p)[1] = make_float4(v[4], v[5], v[6], v[7]);
}

__host__ __device__ constexpr int delta_rows_ld(int DP) { return DP + 8; }      // floats of a token's row in LDS
constexpr int kTokLd = kDeltaChunk + 4;                                          // floats of a row that runs over the tokens
__host__ __device__ constexpr int delta_region(int DP) {                         // C rows over d, or d rows over the tokens
  return kDeltaChunk * delta_rows_ld(DP) > DP * kTokLd ? kDeltaChunk * delta_rows_ld(DP) : DP * kTokLd;
}
static size_t delta_chunk_lds(int DP) { return (size_t)(5 * delta_region(DP) + 4 * kDeltaChunk * kTokLd + 5 * DP) * sizeof(float); }

template <typename T>
__global__ __launch_bounds__(256) void delta_chunk_kernel(DeltaArgs a, DeltaChunks ck, int vec) {
  extern __shared__ float4 lds_raw[];
  constexpr int C = kDeltaChunk;
  const int DT = ck.DT, DP = 16 * DT, LD = delta_rows_ld(DP), region = delta_region(DP);
  float* U = reinterpret_cast<float*>(lds_raw);      // [C][LD]; then U'^T [DP][kTokLd]
  float* R = U + region;                             // [C][LD]
  float* K = R + region;                             // [C][LD]: k, k / G; then L_k V [C][LD]
  float* B = K + region;                             // [C][LD]: b, b / G; then V'^T [DP][kTokLd]
  float* V = B + region;                             // V^T [DP][kTokLd]
  float* mats = V + region;                          // L_k, L_b, A_k, -A_b [C][kTokLd] each; before that the decays' logarithms [C][LD]
  float* totals = mats + 4 * C * kTokLd;             // [4][DP] sums of the logarithms over eight tokens, then [DP] G_C
  float* gC = totals + 4 * DP;
  const int head = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, d = a.d;
  int seq, local;
  if (!delta_chunk_of(a.cu_seqlens, ck.num_seqs, blockIdx.y, seq, local)) return;
  const int first = a.cu_seqlens[seq] + local * C, L = min(C, a.cu_seqlens[seq + 1] - first);
  const size_t ch = (size_t)blockIdx.y * a.heads + head;
  float* logs = mats;
  {
    // eight threads to a token: unit key, removal direction, logarithm of the decay
    const int t = tid >> 3, s = tid & 7;
    const bool on = t < L;
    const T* row = reinterpret_cast<const T*>(a.rows) + (size_t)(first + (on ? t : 0)) * a.stride + (size_t)head * d;
    const float* raw_w = a.raw_w + (size_t)(first + (on ? t : 0)) * a.w_stride + (size_t)head * d;
    float sq = 0.f;
    if (vec) {
      // eight neighbouring elements to a thread and load
      for (int n = 8 * s; n < DP; n += 64) {
        float k[8], r[8], v[8], ra[8], rw[8];
        load8(row + a.k_at + n, k, on); load8(row + a.r_at + n, r, on); load8(row + a.v_at + n, v, on); load8(row + a.a_at + n, ra, on);
        load8(raw_w + n, rw, on);
        float w0[8], ba[8];
        load8(a.w0 + (size_t)head * d + n, w0, true); load8(a.bias_a + (size_t)head * d + n, ba, true);
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          sq = fmaf(k[e], k[e], sq);
          V[(n + e) * kTokLd + t] = v[e];
          rw[e] = on ? -kDecayRate * sigmoid_f32(rw[e] + w0[e]) : 0.f;
          ra[e] = on ? sigmoid_f32(ra[e] + ba[e]) : 0.f;
        }
        store8(K + t * LD + n, k); store8(R + t * LD + n, r); store8(logs + t * LD + n, rw); store8(B + t * LD + n, ra);
      }
    } else
    for (int n = s; n < DP; n += 8) {
      const bool in = on && n < d;
      const float k = in ? to_f32(row[a.k_at + n]) : 0.f;
      K[t * LD + n] = k;
      sq = fmaf(k, k, sq);
      R[t * LD + n] = in ? to_f32(row[a.r_at + n]) : 0.f;
      V[n * kTokLd + t] = in ? to_f32(row[a.v_at + n]) : 0.f;
      logs[t * LD + n] = in ? -kDecayRate * sigmoid_f32(raw_w[n] + a.w0[(size_t)head * d + n]) : 0.f;
      B[t * LD + n] = in ? sigmoid_f32(to_f32(row[a.a_at + n]) + a.bias_a[(size_t)head * d + n]) : 0.f;
    }
#pragma unroll
    for (int off = 1; off < 8; off <<= 1) sq += __shfl_xor(sq, off, 64);
    const float inv = 1.f / sqrtf(sq + kUnitEps);
    for (int n = vec ? 8 * s : s; n < DP; n += vec ? 64 : 8)
     for (int e = 0; e < (vec ? 8 : 1); ++e) {
      const float u = K[t * LD + n + e] * inv;
      U[t * LD + n + e] = u;
      B[t * LD + n + e] *= u;
    }
  }
  __syncthreads();
  // sums of the logarithms over the tokens, eight tokens to a thread
  for (int idx = tid; idx < 4 * DP; idx += 256) {
    const int n = idx % DP, q = idx / DP;
    float sum = 0.f;
#pragma unroll
    for (int t = 0; t < 8; ++t) sum += logs[(8 * q + t) * LD + n];
    totals[q * DP + n] = sum;
  }
  __syncthreads();
  for (int idx = tid; idx < 4 * DP; idx += 256) {
    const int n = idx % DP, q = idx / DP;
    float sum = 0.f;
    for (int p = 0; p < q; ++p) sum += totals[p * DP + n];
#pragma unroll
    for (int t = 0; t < 8; ++t) {
      const int at = (8 * q + t) * LD + n;
      U[at] *= expf(sum);
      sum += logs[at];
      const float up = expf(sum), down = expf(-sum);
      R[at] *= up;
      K[at] *= down;
      B[at] *= down;
      if (8 * q + t == C - 1) gC[n] = up;
    }
  }
  __syncthreads();
  const int g = lane >> 4, m = lane & 15;
  const delta_floatx4 zero = {0.f, 0.f, 0.f, 0.f};
  {
    // wavefront 0: L_k, 1: L_b, 2: A_k, 3: -A_b; tiles (0, 0), (1, 0), (1, 1), the fourth is zero
    const float* left = wave < 2 ? U : R;
    const float* right = (wave & 1) ? B : K;
    delta_floatx4 acc[3] = {zero, zero, zero};
    for (int kb = 0; kb < DT; ++kb) {
      const int at = 16 * kb + 4 * g;
      const delta_floatx4 l0 = lds4(left + m * LD + at), l1 = lds4(left + (16 + m) * LD + at);
      const delta_floatx4 r0 = lds4(right + m * LD + at), r1 = lds4(right + (16 + m) * LD + at);
      acc[0] = mfma4(l0, r0, acc[0]);
      acc[1] = mfma4(l1, r0, acc[1]);
      acc[2] = mfma4(l1, r1, acc[2]);
    }
    float* out = mats + wave * C * kTokLd;           // (the logarithms there were used up in front of the barrier)
    const float sign = wave == 3 ? -1.f : 1.f;
    const int keep = wave < 2 ? 0 : 1;               // j < t, or j <= t
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int r = 4 * g + i;
      out[r * kTokLd + m] = m < r + keep ? sign * acc[0][i] : 0.f;
      out[r * kTokLd + 16 + m] = 0.f;
      out[(16 + r) * kTokLd + m] = sign * acc[1][i];
      out[(16 + r) * kTokLd + 16 + m] = m < r + keep ? sign * acc[2][i] : 0.f;
    }
  }
  // K'^T and B'^T, V and G_C for the second kernel
  for (int f = wave; f < 4 * DT; f += 4) {
    const int tile = f >> 2, part = f & 3, n = 16 * tile + m, t = 16 * (part & 1) + 4 * g;
    const float* x = part < 2 ? K : B;
    const float scale = part < 2 ? gC[n] : -gC[n];
    delta_floatx4 v;
#pragma unroll
    for (int i = 0; i < 4; ++i) v[i] = x[(t + i) * LD + n] * scale;
    *reinterpret_cast<delta_floatx4*>(ck.kb + ((ch * DT * 4 + f) * 64 + lane) * 4) = v;
  }
  for (int f = wave; f < 2 * DT; f += 4)
    *reinterpret_cast<delta_floatx4*>(ck.vf + ((ch * DT * 2 + f) * 64 + lane) * 4) = lds4(V + (16 * (f >> 1) + m) * kTokLd + 16 * (f & 1) + 4 * g);
  for (int n = tid; n < DP; n += 256) ck.gamma[ch * DP + n] = gC[n];
  __syncthreads();
  const float* Lk = mats;
  const float* Lb = mats + C * kTokLd;
  const float* Ak = mats + 2 * C * kTokLd;
  const float* Ab = mats + 3 * C * kTokLd;
  float* W = K;
  for (int f = wave; f < 2 * DT; f += 4) {           // L_k V
    const int rt = f & 1, ct = f >> 1;
    delta_floatx4 acc = zero;
    for (int kb = 0; kb <= rt; ++kb) acc = mfma4(lds4(Lk + (16 * rt + m) * kTokLd + 16 * kb + 4 * g), lds4(V + (16 * ct + m) * kTokLd + 16 * kb + 4 * g), acc);
#pragma unroll
    for (int i = 0; i < 4; ++i) W[(16 * rt + 4 * g + i) * LD + 16 * ct + m] = acc[i];
  }
  __syncthreads();
  // (I + L_b) [U' | V'] = [U | L_k V], a thread per column
  const bool solves = tid < 2 * DP;
  float x[C];
  if (solves) {
    const float* src = tid < DP ? U + tid : W + (tid - DP);
#pragma unroll
    for (int t = 0; t < C; ++t) x[t] = src[t * LD];
#pragma unroll
    for (int t = 1; t < C; ++t) {
      float acc[4] = {x[t], 0.f, 0.f, 0.f};
#pragma unroll
      for (int j = 0; j < C; j += 4)
        if (j < t) {
          const delta_floatx4 l = lds4(Lb + t * kTokLd + j);     // (elements from t on are zero)
#pragma unroll
          for (int e = 0; e < 4; ++e)
            if (j + e < t) acc[e] = fmaf(-l[e], x[j + e], acc[e]);
        }
      x[t] = (acc[0] + acc[1]) + (acc[2] + acc[3]);
    }
  }
  __syncthreads();                                   // every column of U and of L_k V has been read
  if (solves) {
    const int n = tid < DP ? tid : tid - DP;
    float* dst = (tid < DP ? U : B) + n * kTokLd;
    float* ur = ck.ur + ch * 4 * DT * 256;
    float* vo = ck.vo + ch * 4 * DT * 256;
#pragma unroll
    for (int t = 0; t < C; t += 4) {
      const delta_floatx4 v = {x[t], x[t + 1], x[t + 2], x[t + 3]};
      *reinterpret_cast<delta_floatx4*>(dst + t) = v;
      if (tid < DP) {
#pragma unroll
        for (int e = 0; e < 4; ++e) ur[(((t + e) >> 4) * DT + (n >> 4)) * 256 + (((n & 15) >> 2) * 16 + ((t + e) & 15)) * 4 + (n & 3)] = v[e];
      } else {
        *reinterpret_cast<delta_floatx4*>(vo + ((t >> 4) * DT + (n >> 4)) * 256 + (((t & 15) >> 2) * 16 + (n & 15)) * 4) = v;
      }
    }
  }
  __syncthreads();
  for (int f = wave; f < 4 * DT; f += 4) {
    const int rt = f & 1, ct = (f >> 1) % DT;
    const bool readout = f >= 2 * DT;                 // R' first, then O'
    delta_floatx4 acc = zero;
    if (!readout) {
#pragma unroll
      for (int i = 0; i < 4; ++i) acc[i] = R[(16 * rt + 4 * g + i) * LD + 16 * ct + m];
    }
    const float* X = readout ? B : U;
    for (int kb = 0; kb <= rt; ++kb) {
      const int left = (16 * rt + m) * kTokLd + 16 * kb + 4 * g, right = (16 * ct + m) * kTokLd + 16 * kb + 4 * g;
      acc = mfma4(lds4(Ab + left), lds4(X + right), acc);
      if (readout) acc = mfma4(lds4(Ak + left), lds4(V + right), acc);
    }
    if (readout) {
      *reinterpret_cast<delta_floatx4*>(ck.vo + ((ch * 4 + 2 + rt) * DT + ct) * 256 + lane * 4) = acc;
    } else {
      float* ur = ck.ur + ((ch * 4 + 2 + rt) * DT + ct) * 256;
#pragma unroll
      for (int i = 0; i < 4; ++i) ur[((m >> 2) * 16 + 4 * g + i) * 4 + (m & 3)] = acc[i];
    }
  }
}

// One workgroup per (block of 16 columns, head, sequence); wavefront w < 4 makes a tile of 16 rows of [Z; O], wavefront w < DT
// keeps 16 rows of S.  The blocks of one head are a multiple of the heads apart in the grid: with a multiple of eight heads
// they run on one XCD and share its L2.
template <int DT>
__global__ __launch_bounds__(DT > 4 ? 512 : 256) void delta_carry_kernel(DeltaArgs a, DeltaChunks ck) {
  __shared__ delta_floatx4 s_frag[DT][64], z_frag[2][64];
  constexpr int C = kDeltaChunk, DP = 16 * DT;
  const int head = blockIdx.x % a.heads, ct = blockIdx.x / a.heads, seq = blockIdx.y, d = a.d;
  const int lane = threadIdx.x & 63, w = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), g = lane >> 4, c = lane & 15;
  const int q_begin = a.cu_seqlens[seq], q_len = a.cu_seqlens[seq + 1] - q_begin;
  if (q_len <= 0) return;                                       // the whole workgroup
  int base = 0;
  for (int s = 0; s < seq; ++s) base += (a.cu_seqlens[s + 1] - a.cu_seqlens[s] + C - 1) / C;
  const int chunks = (q_len + C - 1) / C;
  const int col = 16 * ct + c;
  float* st = a.state + (size_t)a.state_slots[seq] * a.slot_stride + (size_t)head * d * d;
  const bool carried = a.seq_starts[seq] > 0, holds = w < DT, reads = w < 4;
  delta_floatx4 S = {0.f, 0.f, 0.f, 0.f};
  if (holds && carried && col < d) {
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (16 * w + 4 * g + i < d) S[i] = st[(size_t)(16 * w + 4 * g + i) * d + col];
  }
  if (holds) s_frag[w][lane] = S;
  struct Operands { delta_floatx4 ur[DT], vo, kb[4], v[2], gamma; };
  auto fetch = [&](int j) {
    Operands o;
    const size_t ch = (size_t)(base + j) * a.heads + head;
    if (reads) {
#pragma unroll
      for (int k = 0; k < DT; ++k) o.ur[k] = *reinterpret_cast<const delta_floatx4*>(ck.ur + ((ch * 4 + w) * DT + k) * 256 + lane * 4);
      o.vo = *reinterpret_cast<const delta_floatx4*>(ck.vo + ((ch * 4 + w) * DT + ct) * 256 + lane * 4);
    }
    if (holds) {
#pragma unroll
      for (int k = 0; k < 4; ++k) o.kb[k] = *reinterpret_cast<const delta_floatx4*>(ck.kb + ((ch * DT + w) * 4 + k) * 256 + lane * 4);
#pragma unroll
      for (int k = 0; k < 2; ++k) o.v[k] = *reinterpret_cast<const delta_floatx4*>(ck.vf + ((ch * DT + ct) * 2 + k) * 256 + lane * 4);
      o.gamma = *reinterpret_cast<const delta_floatx4*>(ck.gamma + ch * DP + 16 * w + 4 * g);
    }
    return o;
  };
  // the operands of two chunks are under way while a third is worked off
  Operands ahead[2];
  ahead[0] = fetch(0);
  if (chunks > 1) ahead[1] = fetch(1);
  __syncthreads();
  auto step = [&](int j, Operands& held) {
    const Operands o = held;
    if (j + 2 < chunks) held = fetch(j + 2);
    if (reads) {
      delta_floatx4 acc = o.vo;
#pragma unroll
      for (int k = 0; k < DT; ++k) acc = mfma4(o.ur[k], s_frag[k][lane], acc);
      if (w < 2) {
        z_frag[w][lane] = acc;
      } else if (col < d) {
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          const int t = j * C + 16 * (w - 2) + 4 * g + i;
          if (t < q_len) ck.y[(size_t)(q_begin + t) * a.heads * d + (size_t)head * d + col] = acc[i];
        }
      }
    }
    if (holds) {
#pragma unroll
      for (int i = 0; i < 4; ++i) S[i] *= o.gamma[i];
      S = mfma4(o.kb[0], o.v[0], S);
      S = mfma4(o.kb[1], o.v[1], S);
    }
    __syncthreads();                                            // Z is there, and nobody reads the old S any more
    if (holds) {
      S = mfma4(o.kb[2], z_frag[0][lane], S);
      S = mfma4(o.kb[3], z_frag[1][lane], S);
      s_frag[w][lane] = S;
    }
    __syncthreads();
  };
  for (int j = 0; j < chunks; j += 2) {
    step(j, ahead[0]);
    if (j + 1 < chunks) step(j + 1, ahead[1]);
  }
  if (holds && col < d) {
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (16 * w + 4 * g + i < d) st[(size_t)(16 * w + 4 * g + i) * d + col] = S[i];
  }
}

// Floats of workspace that pllm_delta_rule_chunks needs per chunk (all heads).
PLLM_API int pllm_delta_chunk_floats(int heads, int d) {
  const int DT = (d + 15) / 16;
  return heads * (256 * DT * (4 + 4 + 4 + 2) + 16 * DT);
}

// Long portions: chunks of 32 tokens; the output is the memory's readout in float, y [T, heads * d], without the norm and the
// gate behind it.  workspace: max_chunks * pllm_delta_chunk_floats floats, 16-byte aligned; max_chunks >= sum over the
// sequences of ceil(q_len / 32).
PLLM_API int pllm_delta_rule_chunks(int dtype, const void* rows, long stride, int r_at, int k_at, int v_at, int a_at, const float* raw_w,
                                    long w_stride, const float* w0, const float* bias_a, float* state, long slot_stride,
                                    const int* state_slots, const int* seq_starts, const int* cu_seqlens, float* y, int num_seqs, int heads,
                                    int d, int max_chunks, float* workspace, hipStream_t stream) {
  if (num_seqs <= 0) return 0;
  if (heads <= 0 || d <= 0 || d > kChunkMaxDim || num_seqs > 65535 || max_chunks <= 0 || max_chunks > 65535 || !workspace) return -2;
  DeltaArgs a{rows, stride, r_at, k_at, v_at, a_at, 0, raw_w, w_stride, w0, bias_a, nullptr, 0.f, state, slot_stride,
              state_slots, seq_starts, cu_seqlens, nullptr, heads, d};
  const int DT = (d + 15) / 16;
  const size_t n = (size_t)max_chunks * heads * DT * 256;
  DeltaChunks ck;
  ck.ur = workspace; ck.vo = ck.ur + 4 * n; ck.kb = ck.vo + 4 * n; ck.vf = ck.kb + 4 * n; ck.gamma = ck.vf + 2 * n;
  ck.y = y; ck.num_seqs = num_seqs; ck.max_chunks = max_chunks; ck.DT = DT;
  const size_t lds = delta_chunk_lds(16 * DT);
  dim3 grid(heads, max_chunks);
  // loads of eight elements: heads without padding, every part of a row on a 16-byte boundary
  const int quantum = dtype == PLLM_F32 ? 4 : 8;
  const bool aligned = (uintptr_t)rows % 16 == 0 && (uintptr_t)raw_w % 16 == 0 && (uintptr_t)w0 % 16 == 0 && (uintptr_t)bias_a % 16 == 0;
  const int vec = d % 16 == 0 && aligned && stride % quantum == 0 && w_stride % 4 == 0 && r_at % quantum == 0 && k_at % quantum == 0 &&
                  v_at % quantum == 0 && a_at % quantum == 0;
#define PLLM_DC(T)                                                                                                                     \
  do {                                                                                                                                 \
    hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(delta_chunk_kernel<T>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds); \
    if (e != hipSuccess) return (int)e;                                                                                                \
    hipLaunchKernelGGL(delta_chunk_kernel<T>, grid, dim3(256), lds, stream, a, ck, vec);                                                    \
  } while (0)
  if (dtype == PLLM_F32) PLLM_DC(float); else PLLM_DC(bf16);
#undef PLLM_DC
  dim3 carry(heads * DT, num_seqs);
  switch (DT) {
#define PLLM_DCARRY(N) case N: hipLaunchKernelGGL((delta_carry_kernel<N>), carry, dim3(N > 4 ? 64 * N : 256), 0, stream, a, ck); break;
    PLLM_DCARRY(1) PLLM_DCARRY(2) PLLM_DCARRY(3) PLLM_DCARRY(4) PLLM_DCARRY(5) PLLM_DCARRY(6) PLLM_DCARRY(7) PLLM_DCARRY(8)
#undef PLLM_DCARRY
  }
  PLLM_RETURN_LAST_ERROR();
}
