// Gated delta rule: linear attention whose state forgets by a scalar per head and token and is corrected towards each
// token's value before it is read:
//   S <- a_t S;   u_t = beta_t (v_t - S^T k_t);   S <- S + k_t u_t^T;   o_t = S^T q_t
// with unit-length queries and keys, the state fp32 and carried per sequence.  Beside the decayed scan (decay_scan.hip),
// whose state only adds what a token brings.
#include "act_types.h"

#include <type_traits>

namespace hymeta {

namespace {

constexpr float kMinLog2 = -1.0e4f;         // a decay of 0 (or an overflowed step size): finite, so that differences of sums stay numbers

template <typename A>
__device__ __forceinline__ float exp2_act(float x) {
  return A::kDtype == HYMETA_F32 ? exp2f(x) : __builtin_amdgcn_exp2f(x);
}

// Token by token.  grid = (heads, sequences, value columns in runs of 256); a thread owns one value column c and keeps
// that column of the state, S[:, c], in registers; q_t and k_t go through LDS, their lengths come out of the same loop.
template <typename A, int DMAX>
__global__ __launch_bounds__(256) void delta_rule_rows_kernel(hymeta_delta_rule_args a, int min_rows, int max_rows) {
  typedef typename A::elem elem;
  __shared__ __attribute__((aligned(16))) float s_q[2][DMAX], s_k[2][DMAX];
  const int h = blockIdx.x, s = blockIdx.y;
  const int c = blockIdx.z * 256 + threadIdx.x;
  const int H = a.num_heads, D = a.head_dim, Dv = a.v_dim;
  const int g = h / (H / a.num_qk_heads);
  const int r0 = a.query_start_loc[s], r1 = a.query_start_loc[s + 1];
  if (r1 - r0 < min_rows || r1 - r0 > max_rows) return;
  const int slot = a.slot_idx[s];
  const bool live = c < Dv;
  float* st = (slot >= 0) ? a.state + ((static_cast<int64_t>(slot) * H + h) * D) * Dv : nullptr;
  float S[DMAX];
  const bool carry = st != nullptr && a.context_lens[s] > 0 && live;
#pragma unroll
  for (int d = 0; d < DMAX; ++d) S[d] = (carry && d < D) ? st[static_cast<int64_t>(d) * Dv + c] : 0.f;
  float* out = static_cast<float*>(a.out);
  for (int t = r0; t < r1; ++t) {
    const elem* q = static_cast<const elem*>(a.q) + static_cast<int64_t>(t) * a.q_stride_t + static_cast<int64_t>(g) * D;
    const elem* k = static_cast<const elem*>(a.k) + static_cast<int64_t>(t) * a.k_stride_t + static_cast<int64_t>(g) * D;
    const int buf = (t - r0) & 1;
    for (int d = threadIdx.x; d < DMAX; d += blockDim.x) {
      s_q[buf][d] = d < D ? A::ld(q + d) : 0.f;
      s_k[buf][d] = d < D ? A::ld(k + d) : 0.f;
    }
    const float v = live ? A::ld(static_cast<const elem*>(a.v) + static_cast<int64_t>(t) * a.v_stride_t + static_cast<int64_t>(h) * Dv + c) : 0.f;
    const float decay = exp2_act<A>(fmaxf(a.log2_decay[static_cast<int64_t>(t) * H + h], kMinLog2));
    const float beta = sigmoid_exact(A::ld(static_cast<const elem*>(a.beta_logit) + static_cast<int64_t>(t) * a.beta_stride_t + h));
    __syncthreads();           // one barrier per token: the next token fills the other buffer
    float dot = 0.f, kk = 0.f, qq = 0.f;
#pragma unroll
    for (int d = 0; d < DMAX; ++d) {           // (columns past D hold zeros)
      const float kd = s_k[buf][d], qd = s_q[buf][d];
      dot = fmaf(S[d], kd, dot);
      kk = fmaf(kd, kd, kk);
      qq = fmaf(qd, qd, qq);
    }
    const float ik = 1.f / sqrtf(kk + a.unit_eps), iq = a.q_scale / sqrtf(qq + a.unit_eps);
    const float u = beta * (v - decay * (dot * ik)) * ik;
    float o = 0.f;
#pragma unroll
    for (int d = 0; d < DMAX; ++d) {
      S[d] = fmaf(decay, S[d], s_k[buf][d] * u);
      o = fmaf(S[d], s_q[buf][d], o);
    }
    if (live) out[static_cast<int64_t>(t) * H * Dv + static_cast<int64_t>(h) * Dv + c] = o * iq;
  }
  if (st != nullptr && live) {
#pragma unroll
    for (int d = 0; d < DMAX; ++d)
      if (d < D) st[static_cast<int64_t>(d) * Dv + c] = S[d];
  }
}

// Sequences with one row (decode).  grid = (heads, sequences), 256 threads over the state in fours of value columns: a
// thread takes the columns 4 c4 .. 4 c4 + 3 of the rows d0, d0 + dstep, ... of S and keeps them in registers (16-byte loads,
// all in flight together).  S^T k and S^T q of the OLD state are reduced over the row groups in one go; what the token's own
// write adds to the output is u (k . q), so the state is read once and written once with one reduction between.  Norm: the
// head's output row goes through its RMS norm, weight and silu gate in the same launch.
constexpr int kStepMaxD = 256, kStepRows = 16;
template <typename A, bool Norm>
__global__ __launch_bounds__(256) void delta_rule_step_kernel(hymeta_delta_rule_args a) {
  typedef typename A::elem elem;
  __shared__ float s_q[kStepMaxD], s_k[kStepMaxD];
  __shared__ __attribute__((aligned(16))) float s_a[256 * 4], s_c[256 * 4];
  __shared__ __attribute__((aligned(16))) float s_u[1024];
  __shared__ float red[4];
  const int h = blockIdx.x, s = blockIdx.y;
  const int t = a.query_start_loc[s];
  if (a.query_start_loc[s + 1] - t != 1) return;
  const int H = a.num_heads, D = a.head_dim, Dv = a.v_dim, Dv4 = Dv / 4;
  const int g = h / (H / a.num_qk_heads);
  const int c4 = threadIdx.x % Dv4, d0 = threadIdx.x / Dv4, dstep = 256 / Dv4, lane = threadIdx.x & 63;
  const int slot = a.slot_idx[s];
  float* st = slot >= 0 ? a.state + ((static_cast<int64_t>(slot) * H + h) * D) * Dv : nullptr;
  const bool carry = st != nullptr && a.context_lens[s] > 0;
  f32x4 S[kStepRows];
#pragma unroll
  for (int u = 0; u < kStepRows; ++u) {
    const int d = d0 + u * dstep;
    S[u] = (carry && d < D) ? *reinterpret_cast<const f32x4*>(st + static_cast<int64_t>(d) * Dv + 4 * c4) : f32x4{0.f, 0.f, 0.f, 0.f};
  }
  const elem* q = static_cast<const elem*>(a.q) + static_cast<int64_t>(t) * a.q_stride_t + static_cast<int64_t>(g) * D;
  const elem* k = static_cast<const elem*>(a.k) + static_cast<int64_t>(t) * a.k_stride_t + static_cast<int64_t>(g) * D;
  const float decay = exp2_act<A>(fmaxf(a.log2_decay[static_cast<int64_t>(t) * H + h], kMinLog2));
  const float beta = sigmoid_exact(A::ld(static_cast<const elem*>(a.beta_logit) + static_cast<int64_t>(t) * a.beta_stride_t + h));
  // every wave sums the lengths and the product for itself
  float kk = 0.f, qq = 0.f, kq = 0.f;
  for (int d = lane; d < D; d += 64) {
    const float kd = A::ld(k + d), qd = A::ld(q + d);
    if (threadIdx.x < 64) s_k[d] = kd, s_q[d] = qd;
    kk = fmaf(kd, kd, kk);
    qq = fmaf(qd, qd, qq);
    kq = fmaf(kd, qd, kq);
  }
  kk = wave_sum(kk), qq = wave_sum(qq), kq = wave_sum(kq);
  const float ik = 1.f / sqrtf(kk + a.unit_eps), iq = a.q_scale / sqrtf(qq + a.unit_eps);
  __syncthreads();
  f32x4 pa = f32x4{0.f, 0.f, 0.f, 0.f}, pc = pa;
#pragma unroll
  for (int u = 0; u < kStepRows; ++u) {
    const int d = d0 + u * dstep;
    if (d >= D) continue;
    const float kd = s_k[d], qd = s_q[d];
#pragma unroll
    for (int e = 0; e < 4; ++e) pa[e] = fmaf(S[u][e], kd, pa[e]), pc[e] = fmaf(S[u][e], qd, pc[e]);
  }
  *reinterpret_cast<f32x4*>(&s_a[threadIdx.x * 4]) = pa;          // [d0][4 c4 + e]
  *reinterpret_cast<f32x4*>(&s_c[threadIdx.x * 4]) = pc;
  __syncthreads();
  float o[4] = {0.f, 0.f, 0.f, 0.f}, ss = 0.f;                    // columns threadIdx.x, + 256, ...
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int c = threadIdx.x + 256 * i;
    if (c >= Dv) continue;
    float da = 0.f, dc = 0.f;
    for (int gg = 0; gg < dstep; ++gg) da += s_a[gg * Dv + c], dc += s_c[gg * Dv + c];
    const float v = A::ld(static_cast<const elem*>(a.v) + static_cast<int64_t>(t) * a.v_stride_t + static_cast<int64_t>(h) * Dv + c);
    const float u = beta * (v - decay * (da * ik)) * ik;          // (with the key's length: what multiplies the raw key)
    s_u[c] = u;
    o[i] = iq * fmaf(u, kq, decay * dc);
    ss = fmaf(o[i], o[i], ss);
  }
  __syncthreads();
  if (st != nullptr) {
    const f32x4 u4 = *reinterpret_cast<const f32x4*>(&s_u[4 * c4]);
#pragma unroll
    for (int u = 0; u < kStepRows; ++u) {
      const int d = d0 + u * dstep;
      if (d >= D) continue;
      const float kd = s_k[d];
#pragma unroll
      for (int e = 0; e < 4; ++e) S[u][e] = fmaf(decay, S[u][e], kd * u4[e]);
      *reinterpret_cast<f32x4*>(st + static_cast<int64_t>(d) * Dv + 4 * c4) = S[u];
    }
  }
  const int64_t at = (static_cast<int64_t>(t) * H + h) * Dv;
  if constexpr (Norm) {
    ss = block_sum<4>(ss, red);
    const float inv = 1.f / sqrtf(ss / static_cast<float>(Dv) + a.norm_eps);
    const elem* gate = static_cast<const elem*>(a.gate) + static_cast<int64_t>(t) * a.gate_stride_t + static_cast<int64_t>(h) * Dv;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int c = threadIdx.x + 256 * i;
      if (c >= Dv) continue;
      const float gv = A::ld(gate + c);
      A::st(static_cast<elem*>(a.out) + at + c, o[i] * inv * a.norm_weight[c] * gv * sigmoid_exact(gv));
    }
  } else {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int c = threadIdx.x + 256 * i;
      if (c < Dv) static_cast<float*>(a.out)[at + c] = o[i];
    }
  }
}

// ------------------------------------------------------------------------------------------------
// bf16 portions in chunks of 64 rows on the matrix cores.  With S the state before the chunk, i and j rows of it, c_i the
// running sums of its log2 decays (c the whole chunk's), k' and q' the unit vectors:
//   (I + A) U = diag(beta) V - diag(beta_i 2^(c_i)) K' S,     A_ij = beta_i 2^(c_i - c_j) (k'_i . k'_j)   for j < i, else 0
//   O = diag(2^(c_i)) Q' S + P U,                             P_ij = 2^(c_i - c_j) (q'_i . k'_j)          for j <= i, else 0
//   S_new = 2^c S + sum_j 2^(c - c_j) k'_j u_j^T
// T = (I + A)^-1 and P depend on the chunk alone: a first launch computes them for all chunks and heads side by side; a
// second one carries the state through a sequence's chunks.  The keys and queries enter every product as the bf16 rows they
// are, their lengths as fp32 factors of the rows around the product; what enters a product from fp32 (T, P, the state, U
// and the right-hand side) goes in as hi + lo bf16 parts, so that it keeps 16 bits of mantissa.
//
// Chunks are numbered so that no count has to be known ahead: chunk c of sequence s is number
// query_start_loc[s] / 64 + s + c, at most num_tokens / 64 + num_seqs of them.
// ------------------------------------------------------------------------------------------------
typedef float f32x4v __attribute__((ext_vector_type(4)));
constexpr int kChunk = HYMETA_DELTA_CHUNK;
// Workgroups (with slices of 32 value columns) up to which the second launch runs slices of 16: measured for one prompt of 8192
// with 28 heads of 128 x 128 (112 workgroups) 357 against 405 us, with 64 heads (256) 706 against 566 us.
constexpr int kFewGroups = 128;
constexpr int kChunkMinRows = 8;            // shorter portions go token by token
constexpr int kMat = kChunk * kChunk;
// Where the second launch reads 64 x 64 matrices (or the chunk's keys) as matrix operands, they lie in the operand's own
// order: per 16 rows and 32 columns the 64 lanes' 8 elements one after the other, so that a wave's load is 1 KB in a row.
__device__ __forceinline__ int operand_at(int row, int col, int cols) {       // (col in whole fours)
  return ((row >> 4) * (cols >> 5) + (col >> 5)) * 512 + (((col >> 3) & 3) * 16 + (row & 15)) * 8 + (col & 7);
}
// a chunk's and head's place in the workspace: T hi, T lo, P hi, P lo (bf16, operand order), then per row beta,
// beta 2^(c_i) / |k|, q_scale 2^(c_i) / |q|, 2^(c - c_j) / |k|, then 2^c
struct ChunkPlace {
  uint16_t t[2][kMat], p[2][kMat];
  float beta[kChunk], rhs[kChunk], read[kChunk], write[kChunk];
  float total, pad[3];
};
static_assert(sizeof(ChunkPlace) % 16 == 0, "16-byte loads of every place");

__device__ __forceinline__ f32x4v mfma16(bf16x8 a, bf16x8 b, f32x4v c) { return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0); }
__device__ __forceinline__ bf16x8 frag(u32x4 v) { return __builtin_bit_cast(bf16x8, v); }

// four fp32 values as hi + lo bf16 parts
__device__ __forceinline__ void split4(const float* v, u32x2& hi, u32x2& lo) {
#pragma unroll
  for (int u = 0; u < 2; ++u) {
    hi[u] = pack_bf16x2(v[2 * u], v[2 * u + 1]);
    lo[u] = pack_bf16x2(v[2 * u] - lo_bf(hi[u]), v[2 * u + 1] - hi_bf(hi[u]));
  }
}

// Workspace: the chunks' places ([chunk][head]), then per chunk and query / key head the chunk's keys [64][D], queries [64][D]
// and transposed keys [D][64], bf16 in operand order.
__host__ __device__ inline size_t rows_at(int64_t chunks, int heads) { return static_cast<size_t>(chunks) * heads * sizeof(ChunkPlace); }

// grid = (chunk numbers, heads), 4 waves with 16 rows of the chunk each.
template <int D>
__global__ __launch_bounds__(256) void delta_chunk_solve_kernel(hymeta_delta_rule_args a, int64_t chunks) {
  constexpr int PK = D + 8, PF = kChunk + 4;
  __shared__ __attribute__((aligned(16))) uint16_t sk[kChunk * PK];
  __shared__ __attribute__((aligned(16))) float sA[kChunk * PF], sT[kChunk * PF];
  __shared__ float s_hi[kChunk], s_lo[kChunk], s_beta[kChunk], s_ik[kChunk], s_iq[kChunk];
  // the sequence: the last one whose first number is not past this one
  const int number = blockIdx.x;
  int s = 0;
  for (int lo = 0, hi = a.num_seqs - 1; lo <= hi;) {
    const int mid = (lo + hi) >> 1;
    if (a.query_start_loc[mid] / kChunk + mid <= number) s = mid, lo = mid + 1;
    else hi = mid - 1;
  }
  const int r0 = a.query_start_loc[s], rows = a.query_start_loc[s + 1] - r0;
  const int c0 = (number - (r0 / kChunk + s)) * kChunk;
  if (rows < kChunkMinRows || c0 >= rows) return;
  const int nrow = min(kChunk, rows - c0), h = blockIdx.y, H = a.num_heads, group = H / a.num_qk_heads, g = h / group;
  const int64_t t0 = r0 + c0;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, n = lane & 15, g4 = lane >> 4;
  const int i = 16 * wave + n;                          // this lane's row of the chunk
  ChunkPlace* place = static_cast<ChunkPlace*>(a.workspace) + static_cast<int64_t>(number) * H + h;
  u32x4 kf[D / 32], qf[D / 32];
  {
    const uint16_t* kr = static_cast<const uint16_t*>(a.k) + (t0 + i) * a.k_stride_t + static_cast<int64_t>(g) * D + 8 * g4;
    const uint16_t* qr = static_cast<const uint16_t*>(a.q) + (t0 + i) * a.q_stride_t + static_cast<int64_t>(g) * D + 8 * g4;
#pragma unroll
    for (int sd = 0; sd < D / 32; ++sd) {
      kf[sd] = qf[sd] = u32x4{0u, 0u, 0u, 0u};
      if (i < nrow) kf[sd] = ld16g(kr + 32 * sd), qf[sd] = ld16g(qr + 32 * sd);
    }
  }
  if (wave == 0) {
    // running sums in double precision, kept as two floats: a difference of two sums is exact to its own rounding however
    // large the sums are
    const bool on = lane < nrow;
    double cum = on ? static_cast<double>(fmaxf(a.log2_decay[(t0 + lane) * H + h], kMinLog2)) : 0.0;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const double up = __shfl_up(cum, o, 64);
      if (lane >= o) cum += up;
    }
    s_hi[lane] = static_cast<float>(cum);
    s_lo[lane] = static_cast<float>(cum - static_cast<double>(s_hi[lane]));
    s_beta[lane] = on ? sigmoid_exact(bf2f(static_cast<const uint16_t*>(a.beta_logit)[(t0 + lane) * a.beta_stride_t + h])) : 0.f;
  }
  float kk = 0.f, qq = 0.f;
#pragma unroll
  for (int sd = 0; sd < D / 32; ++sd) {
    st16(&sk[i * PK + 32 * sd + 8 * g4], kf[sd]);
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      kk = fmaf(lo_bf(kf[sd][u]), lo_bf(kf[sd][u]), fmaf(hi_bf(kf[sd][u]), hi_bf(kf[sd][u]), kk));
      qq = fmaf(lo_bf(qf[sd][u]), lo_bf(qf[sd][u]), fmaf(hi_bf(qf[sd][u]), hi_bf(qf[sd][u]), qq));
    }
  }
  kk += __shfl_xor(kk, 16, 64), kk += __shfl_xor(kk, 32, 64);
  qq += __shfl_xor(qq, 16, 64), qq += __shfl_xor(qq, 32, 64);
  if (g4 == 0) {
    s_ik[i] = 1.f / sqrtf(kk + a.unit_eps);
    s_iq[i] = a.q_scale / sqrtf(qq + a.unit_eps);
  }
  __syncthreads();
  // A and P in blocks of 16 x 16, transposed products: a lane gets four consecutive j of its row i
  const float ch = s_hi[i], cl = s_lo[i], bk = s_beta[i] * s_ik[i], iq = s_iq[i];
#pragma unroll
  for (int jb = 0; jb < 4; ++jb) {
    float av[4] = {0.f, 0.f, 0.f, 0.f}, pv[4] = {0.f, 0.f, 0.f, 0.f};
    if (jb <= wave) {
      f32x4v xk = f32x4v{0.f, 0.f, 0.f, 0.f}, xq = xk;
#pragma unroll
      for (int sd = 0; sd < D / 32; ++sd) {
        const bf16x8 kj = frag(ld16(&sk[(16 * jb + n) * PK + 32 * sd + 8 * g4]));
        xk = mfma16(kj, frag(kf[sd]), xk);
        xq = mfma16(kj, frag(qf[sd]), xq);
      }
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int j = 16 * jb + 4 * g4 + r;
        if (j > i) continue;
        const float w = __builtin_amdgcn_exp2f((ch - s_hi[j]) + (cl - s_lo[j])) * s_ik[j];
        if (j < i) av[r] = bk * w * xk[r];
        pv[r] = iq * w * xq[r];
      }
      *reinterpret_cast<f32x4v*>(&sA[i * PF + 16 * jb + 4 * g4]) = f32x4v{av[0], av[1], av[2], av[3]};
    }
    // (the blocks behind the diagonal are stored as zeros: every wave multiplies all 64 rows)
    u32x2 hi, lo;
    split4(pv, hi, lo);
    *reinterpret_cast<u32x2*>(&place->p[0][operand_at(i, 16 * jb + 4 * g4, kChunk)]) = hi;
    *reinterpret_cast<u32x2*>(&place->p[1][operand_at(i, 16 * jb + 4 * g4, kChunk)]) = lo;
  }
  __syncthreads();
  // T: the diagonal blocks by forward substitution, a column per lane (the four groups of lanes do the same)
  {
    float x[16];
#pragma unroll
    for (int r = 0; r < 16; ++r) {
      float v = r == n ? 1.f : 0.f;
#pragma unroll
      for (int j = 0; j < r; ++j) v = fmaf(-sA[(16 * wave + r) * PF + 16 * wave + j], x[j], v);
      x[r] = v;
    }
    if (g4 == 0) {
#pragma unroll
      for (int r = 0; r < 16; ++r) sT[(16 * wave + r) * PF + 16 * wave + n] = x[r];
    }
  }
  __syncthreads();
  // ... then the blocks below them, a diagonal at a time: T_ij = -T_ii sum_{j <= l < i} A_il T_lj, in fp32 on the matrix
  // cores (step e of a product takes the inner indices 4 g4 + e, so that the first product's result is the second's operand
  // as it lies in the registers)
#pragma unroll
  for (int below = 1; below < 4; ++below) {
    if (wave >= below) {
      const int jb = wave - below;
      f32x4v m = f32x4v{0.f, 0.f, 0.f, 0.f}, x = m;
      for (int lb = jb; lb < wave; ++lb) {
        const f32x4v al = *reinterpret_cast<const f32x4v*>(&sA[i * PF + 16 * lb + 4 * g4]);
#pragma unroll
        for (int e = 0; e < 4; ++e) m = __builtin_amdgcn_mfma_f32_16x16x4f32(al[e], sT[(16 * lb + 4 * g4 + e) * PF + 16 * jb + n], m, 0, 0, 0);
      }
      const f32x4v ti = *reinterpret_cast<const f32x4v*>(&sT[i * PF + 16 * wave + 4 * g4]);
#pragma unroll
      for (int e = 0; e < 4; ++e) x = __builtin_amdgcn_mfma_f32_16x16x4f32(ti[e], m[e], x, 0, 0, 0);
#pragma unroll
      for (int r = 0; r < 4; ++r) sT[(16 * wave + 4 * g4 + r) * PF + 16 * jb + n] = -x[r];
    }
    __syncthreads();
  }
  {
    const int row = tid >> 2, jb = tid & 3, rb = row >> 4;
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      float v[4] = {0.f, 0.f, 0.f, 0.f};
      if (jb <= rb) {
        const f32x4v tv = *reinterpret_cast<const f32x4v*>(&sT[row * PF + 16 * jb + 4 * u]);
#pragma unroll
        for (int e = 0; e < 4; ++e) v[e] = tv[e];
      }
      u32x2 hi, lo;
      split4(v, hi, lo);
      *reinterpret_cast<u32x2*>(&place->t[0][operand_at(row, 16 * jb + 4 * u, kChunk)]) = hi;
      *reinterpret_cast<u32x2*>(&place->t[1][operand_at(row, 16 * jb + 4 * u, kChunk)]) = lo;
    }
  }
  if (h % group == 0) {
    uint16_t* kr = reinterpret_cast<uint16_t*>(static_cast<char*>(a.workspace) + rows_at(chunks, H)) +
                   (static_cast<int64_t>(number) * a.num_qk_heads + g) * 3 * D * kChunk;
    uint16_t *qr = kr + D * kChunk, *kt = qr + D * kChunk;
#pragma unroll
    for (int sd = 0; sd < D / 32; ++sd) {
      st16(kr + operand_at(i, 32 * sd + 8 * g4, D), kf[sd]);
      st16(qr + operand_at(i, 32 * sd + 8 * g4, D), qf[sd]);
    }
    for (int idx = tid; idx < D * (kChunk / 8); idx += 256) {
      const int d = idx % D, tc = idx / D;
      u32x4 w;
#pragma unroll
      for (int u = 0; u < 4; ++u)
        w[u] = static_cast<uint32_t>(sk[(8 * tc + 2 * u) * PK + d]) | (static_cast<uint32_t>(sk[(8 * tc + 2 * u + 1) * PK + d]) << 16);
      st16(kt + operand_at(d, 8 * tc, kChunk), w);
    }
  }
  if (wave == 0) {
    const float th = s_hi[kChunk - 1], tl = s_lo[kChunk - 1];          // (rows past the portion add 0)
    const float here = __builtin_amdgcn_exp2f(s_hi[lane] + s_lo[lane]);
    place->beta[lane] = s_beta[lane];
    place->rhs[lane] = s_beta[lane] * s_ik[lane] * here;
    place->read[lane] = s_iq[lane] * here;
    place->write[lane] = lane < nrow ? s_ik[lane] * __builtin_amdgcn_exp2f((th - s_hi[lane]) + (tl - s_lo[lane])) : 0.f;
    if (lane == 0) place->total = __builtin_amdgcn_exp2f(th + tl);
  }
}

// grid = (heads, sequences, value columns in slices of 16 CB), 4 waves.  The state slice stays fp32 in registers in blocks of
// 16 x 16 dealt over the waves (a lane holds 4 consecutive rows d of one column); its bf16 parts, the right-hand side and
// U pass through LDS with the reduced index consecutive; everything a chunk brings comes from memory in the matrix
// operands' own layout, loaded two chunks ahead (the loads of two chunks are in flight, each in registers of its own).  Rows past the portion read its last row (beta, and with it what they would
// write, is 0 there), and the last chunk fetches itself once more, so that no load stands under a condition.
template <int D, int CB>
__global__ __launch_bounds__(256) void delta_chunk_scan_kernel(hymeta_delta_rule_args a, int64_t chunks) {
  constexpr int SV = 16 * CB, PK = D + 8, PT = kChunk + 8, NBW = (D / 16) * CB / 4;
  static_assert((D / 16) * CB % 4 == 0, "the state's blocks deal evenly over the waves");
  __shared__ __attribute__((aligned(16))) uint16_t sst[2][SV * PK];                                      // state, [c][d]
  __shared__ __attribute__((aligned(16))) uint16_t srt[2][SV * PT], su[2][SV * PT], sw[2][SV * PT];      // [c][row]
  const int h = blockIdx.x, s = blockIdx.y, vs = blockIdx.z;
  const int r0 = a.query_start_loc[s], rows = a.query_start_loc[s + 1] - r0;
  if (rows < kChunkMinRows) return;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, n = lane & 15, g4 = lane >> 4;
  const int H = a.num_heads, G = a.num_qk_heads, Dv = a.v_dim, g = h / (H / G);
  const int slot = a.slot_idx[s];
  float* st = slot >= 0 ? a.state + ((static_cast<int64_t>(slot) * H + h) * D) * Dv + vs * SV : nullptr;
  const bool carry = st != nullptr && a.context_lens[s] > 0;
  f32x4v S[NBW];
#pragma unroll
  for (int ib = 0; ib < NBW; ++ib) {
    const int b = wave + 4 * ib, cb = b % CB, db = b / CB;
#pragma unroll
    for (int r = 0; r < 4; ++r) S[ib][r] = carry ? st[static_cast<int64_t>(16 * db + 4 * g4 + r) * Dv + 16 * cb + n] : 0.f;
  }
  auto state_to_lds = [&]() {
#pragma unroll
    for (int ib = 0; ib < NBW; ++ib) {
      const int b = wave + 4 * ib, cb = b % CB, db = b / CB;
      const float v[4] = {S[ib][0], S[ib][1], S[ib][2], S[ib][3]};
      u32x2 hi, lo;
      split4(v, hi, lo);
      *reinterpret_cast<u32x2*>(&sst[0][(16 * cb + n) * PK + 16 * db + 4 * g4]) = hi;
      *reinterpret_cast<u32x2*>(&sst[1][(16 * cb + n) * PK + 16 * db + 4 * g4]) = lo;
    }
  };
  state_to_lds();
  const uint16_t* vp = static_cast<const uint16_t*>(a.v) + static_cast<int64_t>(h) * Dv + vs * SV + n;
  const int64_t first = r0 / kChunk + s;
  const ChunkPlace* places = static_cast<const ChunkPlace*>(a.workspace) + first * H + h;
  const uint16_t* packed = reinterpret_cast<const uint16_t*>(static_cast<const char*>(a.workspace) + rows_at(chunks, H)) +
                           (first * G + g) * 3 * D * kChunk + 8 * lane;          // keys, queries, transposed keys of the chunks
  const int iq = 16 * wave + 4 * g4;        // the first of the four rows of this lane's results
  // what a chunk brings: row fragments of the keys, queries, T and P, the transposed keys of this wave's state blocks, values
  struct Chunk {
    u32x4 kf[D / 32], qf[D / 32], tf[2][2], pf[2][2], wf[NBW][2];
    uint16_t vv[CB][4];
    f32x4v beta, rhs, read, write;
    float total;
  };
  auto fetch_rows = [&](Chunk& m, int c) {
    const int last = rows - 1 - c * kChunk;
    const int64_t t0 = r0 + static_cast<int64_t>(c) * kChunk;
    const uint16_t* kr = packed + static_cast<int64_t>(c) * G * 3 * D * kChunk + wave * (D / 32) * 512;
#pragma unroll
    for (int sd = 0; sd < D / 32; ++sd) m.kf[sd] = ld16g(kr + 512 * sd), m.qf[sd] = ld16g(kr + D * kChunk + 512 * sd);
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const uint16_t* vr = vp + (t0 + min(iq + r, last)) * a.v_stride_t;
#pragma unroll
      for (int cb = 0; cb < CB; ++cb) m.vv[cb][r] = vr[16 * cb];
    }
  };
  auto fetch_t = [&](Chunk& m, int c) {
    const ChunkPlace* p = places + static_cast<int64_t>(c) * H;
#pragma unroll
    for (int part = 0; part < 2; ++part)
#pragma unroll
      for (int kk = 0; kk < 2; ++kk) m.tf[part][kk] = ld16g(&p->t[part][(2 * wave + kk) * 512 + 8 * lane]);
    m.beta = *reinterpret_cast<const f32x4v*>(&p->beta[iq]);
    m.rhs = *reinterpret_cast<const f32x4v*>(&p->rhs[iq]);
    m.read = *reinterpret_cast<const f32x4v*>(&p->read[iq]);
    m.write = *reinterpret_cast<const f32x4v*>(&p->write[iq]);
  };
  auto fetch_p = [&](Chunk& m, int c) {
    const ChunkPlace* p = places + static_cast<int64_t>(c) * H;
#pragma unroll
    for (int part = 0; part < 2; ++part)
#pragma unroll
      for (int kk = 0; kk < 2; ++kk) m.pf[part][kk] = ld16g(&p->p[part][(2 * wave + kk) * 512 + 8 * lane]);
  };
  auto fetch_transposed = [&](Chunk& m, int c) {
    const uint16_t* kt = packed + (static_cast<int64_t>(c) * G * 3 + 2) * D * kChunk;
    m.total = places[static_cast<int64_t>(c) * H].total;
#pragma unroll
    for (int ib = 0; ib < NBW; ++ib) {
      const int db = (wave + 4 * ib) / CB;
#pragma unroll
      for (int kk = 0; kk < 2; ++kk) m.wf[ib][kk] = ld16g(kt + (2 * db + kk) * 512);
    }
  };
  float* out = static_cast<float*>(a.out) + static_cast<int64_t>(r0) * H * Dv + static_cast<int64_t>(h) * Dv + vs * SV + n;
  const int num = (rows + kChunk - 1) / kChunk;
  auto advance = [&](Chunk& m, int c, auto full) {         // full: a whole chunk (every row is the portion's)
    const int next = min(c + 2, num - 1);
    __syncthreads();                        // the state's parts are in place
    f32x4v x[CB], y[CB];
#pragma unroll
    for (int cb = 0; cb < CB; ++cb) {
      x[cb] = y[cb] = f32x4v{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int sd = 0; sd < D / 32; ++sd) {
        const bf16x8 sh = frag(ld16(&sst[0][(16 * cb + n) * PK + 32 * sd + 8 * g4]));
        const bf16x8 sl = frag(ld16(&sst[1][(16 * cb + n) * PK + 32 * sd + 8 * g4]));
        x[cb] = mfma16(frag(m.kf[sd]), sh, x[cb]);
        y[cb] = mfma16(frag(m.qf[sd]), sh, y[cb]);
        x[cb] = mfma16(frag(m.kf[sd]), sl, x[cb]);
        y[cb] = mfma16(frag(m.qf[sd]), sl, y[cb]);
      }
    }
#pragma unroll
    for (int cb = 0; cb < CB; ++cb) {
      float v[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        v[r] = m.beta[r] * bf2f(m.vv[cb][r]) - m.rhs[r] * x[cb][r];
        y[cb][r] *= m.read[r];
      }
      u32x2 hi, lo;
      split4(v, hi, lo);
      *reinterpret_cast<u32x2*>(&srt[0][(16 * cb + n) * PT + iq]) = hi;
      *reinterpret_cast<u32x2*>(&srt[1][(16 * cb + n) * PT + iq]) = lo;
    }
    fetch_rows(m, next);
    __syncthreads();
#pragma unroll
    for (int cb = 0; cb < CB; ++cb) {
      f32x4v u = f32x4v{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int kk = 0; kk < 2; ++kk) {
        const bf16x8 rh = frag(ld16(&srt[0][(16 * cb + n) * PT + 32 * kk + 8 * g4]));
        const bf16x8 rl = frag(ld16(&srt[1][(16 * cb + n) * PT + 32 * kk + 8 * g4]));
        u = mfma16(frag(m.tf[0][kk]), rh, u);
        u = mfma16(frag(m.tf[0][kk]), rl, u);
        u = mfma16(frag(m.tf[1][kk]), rh, u);
      }
      float v[4] = {u[0], u[1], u[2], u[3]};
      u32x2 hi, lo;
      split4(v, hi, lo);
      *reinterpret_cast<u32x2*>(&su[0][(16 * cb + n) * PT + iq]) = hi;
      *reinterpret_cast<u32x2*>(&su[1][(16 * cb + n) * PT + iq]) = lo;
#pragma unroll
      for (int r = 0; r < 4; ++r) v[r] *= m.write[r];
      split4(v, hi, lo);
      *reinterpret_cast<u32x2*>(&sw[0][(16 * cb + n) * PT + iq]) = hi;
      *reinterpret_cast<u32x2*>(&sw[1][(16 * cb + n) * PT + iq]) = lo;
    }
    fetch_t(m, next);
    __syncthreads();
#pragma unroll
    for (int ib = 0; ib < NBW; ++ib) {
      const int cb = (wave + 4 * ib) % CB;
      f32x4v acc = S[ib] * m.total;
#pragma unroll
      for (int kk = 0; kk < 2; ++kk) {
        acc = mfma16(frag(m.wf[ib][kk]), frag(ld16(&sw[0][(16 * cb + n) * PT + 32 * kk + 8 * g4])), acc);
        acc = mfma16(frag(m.wf[ib][kk]), frag(ld16(&sw[1][(16 * cb + n) * PT + 32 * kk + 8 * g4])), acc);
      }
      S[ib] = acc;
    }
    fetch_transposed(m, next);
    state_to_lds();                         // (its last readers passed the barrier before)
#pragma unroll
    for (int cb = 0; cb < CB; ++cb) {
#pragma unroll
      for (int kk = 0; kk < 2; ++kk) {
        const bf16x8 uh = frag(ld16(&su[0][(16 * cb + n) * PT + 32 * kk + 8 * g4]));
        const bf16x8 ul = frag(ld16(&su[1][(16 * cb + n) * PT + 32 * kk + 8 * g4]));
        y[cb] = mfma16(frag(m.pf[0][kk]), uh, y[cb]);
        y[cb] = mfma16(frag(m.pf[0][kk]), ul, y[cb]);
        y[cb] = mfma16(frag(m.pf[1][kk]), uh, y[cb]);
      }
    }
    fetch_p(m, next);
    const int live = rows - c * kChunk - iq;            // rows of this lane's four that are the portion's
    float* to = out + (static_cast<int64_t>(c) * kChunk + iq) * H * Dv;
#pragma unroll
    for (int r = 0; r < 4; ++r)
      if (decltype(full)::value || r < live) {
#pragma unroll
        for (int cb = 0; cb < CB; ++cb) to[static_cast<int64_t>(r) * H * Dv + 16 * cb] = y[cb][r];
      }
  };
  Chunk even, odd;
  auto fetch = [&](Chunk& m, int c) {
    fetch_rows(m, c);
    fetch_t(m, c);
    fetch_transposed(m, c);
    fetch_p(m, c);
  };
  fetch(even, 0);
  fetch(odd, min(1, num - 1));
  // (the loop's body has no branch: loads under one, or a chunk that might not run, would make the waits in front of the
  // matrix products wait for the loads of the chunks behind as well)
  int c = 0;
  for (; c + 2 < num; c += 2) {
    advance(even, c, std::true_type{});
    advance(odd, c + 1, std::true_type{});
  }
  advance(even, c, std::false_type{});
  if (c + 1 < num) advance(odd, c + 1, std::false_type{});
  if (st != nullptr) {
#pragma unroll
    for (int ib = 0; ib < NBW; ++ib) {
      const int b = wave + 4 * ib, cb = b % CB, db = b / CB;
#pragma unroll
      for (int r = 0; r < 4; ++r) st[static_cast<int64_t>(16 * db + 4 * g4 + r) * Dv + 16 * cb + n] = S[ib][r];
    }
  }
}

inline bool chunk_dims(int head_dim, int v_dim, int act_dtype) {
  return act_dtype == HYMETA_BF16 && head_dim >= 32 && head_dim <= 128 && head_dim % 32 == 0 && v_dim % 32 == 0 && v_dim / 16 <= 65535;
}
inline bool chunk_shape(const hymeta_delta_rule_args& a) {
  auto aligned = [](const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; };
  return chunk_dims(a.head_dim, a.v_dim, a.act_dtype) && a.q_stride_t % 8 == 0 && a.k_stride_t % 8 == 0 && aligned(a.q) && aligned(a.k);
}
inline int64_t chunk_numbers(int num_tokens, int num_seqs) { return static_cast<int64_t>(num_tokens) / kChunk + num_seqs; }

inline bool step_shape(const hymeta_delta_rule_args& a) {
  const int dv4 = a.v_dim / 4;
  return a.v_dim % 4 == 0 && dv4 <= 256 && 256 % dv4 == 0 && a.head_dim <= kStepMaxD && static_cast<int64_t>(a.head_dim) * dv4 <= 256 * kStepRows &&
         reinterpret_cast<uintptr_t>(a.state) % 16 == 0;
}

template <typename A>
void launch_rows(const hymeta_delta_rule_args& a, hipStream_t st, int min_rows, int max_rows) {
  const dim3 grid(a.num_heads, a.num_seqs, (a.v_dim + 255) / 256);
  const dim3 block(a.v_dim >= 256 ? 256 : (a.v_dim + 63) / 64 * 64);
  if (a.head_dim <= 32) hipLaunchKernelGGL((delta_rule_rows_kernel<A, 32>), grid, block, 0, st, a, min_rows, max_rows);
  else if (a.head_dim <= 64) hipLaunchKernelGGL((delta_rule_rows_kernel<A, 64>), grid, block, 0, st, a, min_rows, max_rows);
  else if (a.head_dim <= 128) hipLaunchKernelGGL((delta_rule_rows_kernel<A, 128>), grid, block, 0, st, a, min_rows, max_rows);
  else hipLaunchKernelGGL((delta_rule_rows_kernel<A, 256>), grid, block, 0, st, a, min_rows, max_rows);
}

template <int D>
void launch_chunks(const hymeta_delta_rule_args& a, hipStream_t st, int64_t chunks) {
  hipLaunchKernelGGL(delta_chunk_solve_kernel<D>, dim3(static_cast<unsigned>(chunks), a.num_heads), dim3(256), 0, st, a, chunks);
  // slices of 32 columns reread a chunk's matrices half as often; slices of 16 double the workgroups where they are few
  if constexpr (D % 64 == 0) {
    if (static_cast<int64_t>(a.num_heads) * a.num_seqs * (a.v_dim / 32) <= kFewGroups) {
      hipLaunchKernelGGL((delta_chunk_scan_kernel<D, 1>), dim3(a.num_heads, a.num_seqs, a.v_dim / 16), dim3(256), 0, st, a, chunks);
      return;
    }
  }
  hipLaunchKernelGGL((delta_chunk_scan_kernel<D, 2>), dim3(a.num_heads, a.num_seqs, a.v_dim / 32), dim3(256), 0, st, a, chunks);
}

}  // namespace

}  // namespace hymeta

using namespace hymeta;

extern "C" size_t hymeta_delta_rule_workspace_bytes(int32_t num_tokens, int32_t num_seqs, int32_t num_heads, int32_t num_qk_heads, int32_t head_dim,
                                                    int32_t v_dim, int32_t act_dtype, int32_t max_query_len) {
  if (num_tokens <= 0 || num_seqs <= 0 || num_heads <= 0 || num_qk_heads <= 0 || max_query_len < kChunkMinRows || !chunk_dims(head_dim, v_dim, act_dtype)) return 0;
  const int64_t chunks = chunk_numbers(num_tokens, num_seqs);
  return rows_at(chunks, num_heads) + static_cast<size_t>(chunks) * num_qk_heads * 3 * head_dim * kChunk * 2;
}

extern "C" int hymeta_delta_rule(const hymeta_delta_rule_args* args, hymeta_stream_t stream) {
  if (!args_ok(args)) return HYMETA_ERR_INVALID_ARG;
  const hymeta_delta_rule_args& a = *args;
  if (a.num_tokens < 0 || a.num_seqs < 0 || a.num_heads <= 0 || a.num_qk_heads <= 0 || a.head_dim <= 0 || a.v_dim <= 0) return HYMETA_ERR_INVALID_ARG;
  if (a.num_heads % a.num_qk_heads != 0) return HYMETA_ERR_INVALID_ARG;
  if (!act_dtype_ok(a.act_dtype)) return HYMETA_ERR_UNSUPPORTED;
  if (a.head_dim > 256 || a.num_seqs > 65535 || a.num_heads > 65535 || a.v_dim > 256 * 65535) return HYMETA_ERR_UNSUPPORTED;
  if (a.num_tokens == 0 || a.num_seqs == 0) return HYMETA_OK;
  if (!a.q || !a.k || !a.v || !a.beta_logit || !a.log2_decay || !a.state || !a.out || !a.query_start_loc || !a.context_lens || !a.slot_idx) return HYMETA_ERR_INVALID_ARG;
  const int64_t qk = static_cast<int64_t>(a.num_qk_heads) * a.head_dim, hv = static_cast<int64_t>(a.num_heads) * a.v_dim;
  if (a.q_stride_t < qk || a.k_stride_t < qk || a.v_stride_t < hv || a.beta_stride_t < a.num_heads) return HYMETA_ERR_INVALID_ARG;
  const bool step = step_shape(a);
  if (a.norm_weight) {
    if (!a.gate || a.gate_stride_t < hv) return HYMETA_ERR_INVALID_ARG;
    if (!step || a.max_query_len != 1 || a.num_tokens != a.num_seqs) return HYMETA_ERR_UNSUPPORTED;
  }
  hipStream_t st = begin_launches(stream);
  const bool bf = a.act_dtype == HYMETA_BF16;
  int max_rows = 0x7fffffff;
  if (chunk_shape(a) && a.max_query_len >= kChunkMinRows) {
    const size_t need = hymeta_delta_rule_workspace_bytes(a.num_tokens, a.num_seqs, a.num_heads, a.num_qk_heads, a.head_dim, a.v_dim, a.act_dtype, a.max_query_len);
    if (!a.workspace || a.workspace_bytes < need || reinterpret_cast<uintptr_t>(a.workspace) % 16 != 0) return HYMETA_ERR_WORKSPACE;
    const int64_t chunks = chunk_numbers(a.num_tokens, a.num_seqs);
    if (a.head_dim == 32) launch_chunks<32>(a, st, chunks);
    else if (a.head_dim == 64) launch_chunks<64>(a, st, chunks);
    else if (a.head_dim == 96) launch_chunks<96>(a, st, chunks);
    else launch_chunks<128>(a, st, chunks);
    max_rows = kChunkMinRows - 1;
  }
  int min_rows = 1;
  if (step) {
    const dim3 grid(a.num_heads, a.num_seqs), block(256);
    if (a.norm_weight) {
      if (bf) hipLaunchKernelGGL((delta_rule_step_kernel<ActBf16, true>), grid, block, 0, st, a);
      else hipLaunchKernelGGL((delta_rule_step_kernel<ActF32, true>), grid, block, 0, st, a);
    } else {
      if (bf) hipLaunchKernelGGL((delta_rule_step_kernel<ActBf16, false>), grid, block, 0, st, a);
      else hipLaunchKernelGGL((delta_rule_step_kernel<ActF32, false>), grid, block, 0, st, a);
    }
    min_rows = 2;
  }
  if (a.max_query_len >= min_rows && max_rows >= min_rows) {
    if (bf) launch_rows<ActBf16>(a, st, min_rows, max_rows);
    else launch_rows<ActF32>(a, st, min_rows, max_rows);
  }
  return launch_status();
}
