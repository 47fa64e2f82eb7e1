// Kernels of hybrid decoder designs with a gated delta rule and with differential attention: the recurrence's operands
// (short convolutions over time with their state, silu, unit vectors, step sizes and decays), the recurrence itself in two
// forms (row by row for decoded tokens and short portions, chunks of 64 rows on the matrix cores for long ones), and the
// combination of two attention maps. Everything here is fp32 (the cumulative logarithms of the decays fp64).
//
// The rule, per head with key width D and value width Dv, state S [D, Dv]:
//   S <- g S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q.
//
// A step's sequences are described by cu_q [B + 1] (row ranges), positions [T], slots [B] (state slot, < 0: none) and
// row_seq [T] (sequence of a row, < 0: padding). A sequence whose first row is at position 0 starts from zeros.
#include "hybrid_common.h"

namespace {

LC_DEVICE float softplusf_(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }

// ---------------------------------------------------------------- operands
// One block per token. proj [T, ld]: q [G*D] | k [G*D] | v [H*Dv] (C channels, convolved, silu) and somewhere behind them the
// step-size logits [H] at column col_b and the decay logits [H] at column col_a. Written (rows of the step, fp32):
//   qk [T, 2, G, Dp]   unit q times qscale, unit k (x / sqrt(sum x^2 + 1e-6)), zero from D on
//   v  [T, H, Dvp]     zero from Dv on
//   gates [T, H]       (beta = sigmoid(b), log g = neg_rate[h] * softplus(a + dt_bias[h]))
//   kq [T, G]          q . k
struct DeltaPrepArgs {
  ConvIn in;
  int col_b, col_a;
  const float* neg_rate;
  const float* dt_bias;
  const int32_t* row_seq;
  const int32_t* cu_q;
  const int32_t* positions;
  const int32_t* slots;
  float* qk;
  float* v;
  float2* gates;
  float* kq;
  int H, G, D, Dp, Dv, Dvp;
  float qscale;
  int T, per_xcd;                // rows, rows per chiplet (neighbouring rows share their inputs, so they share an L2)
};

__global__ __launch_bounds__(256) void delta_prep_kernel(DeltaPrepArgs a) {
  extern __shared__ float u[];                       // [C] the token's channels
  const int H = a.H, G = a.G, D = a.D, Dv = a.Dv;
  const int t0 = (blockIdx.x & 7) * a.per_xcd + (blockIdx.x >> 3);   // (workgroups go round robin over the 8 chiplets)
  if (t0 >= a.T) return;
  const int hist = a.in.taps > 1 ? a.in.taps - 1 : 0;
  const RowSeq s = row_sequence(t0, a.row_seq, a.cu_q, a.positions, a.slots);
  const int count = conv_rows_of_block(t0, s, hist);
  if (count == 0) return;                            // served by the portion's first row
  float* st = s.slot >= 0 && hist > 0 ? a.in.state + static_cast<size_t>(s.slot) * a.in.state_stride : nullptr;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  for (int rr = 0; rr < count; ++rr) {
    const size_t t = t0 + rr;
    conv_token<true>(a.in, s, st, static_cast<int>(t) - s.first, u);
    const float* row = a.in.x + t * a.in.ld;
    for (int h = threadIdx.x; h < H; h += 256)
      a.gates[t * H + h] = make_float2(sigmoidf_(row[a.col_b + h]), a.neg_rate[h] * softplusf_(row[a.col_a + h] + a.dt_bias[h]));
    __syncthreads();
    for (int g = wave; g < G; g += 4) {              // a wave owns a q head and its k head
      const float* q = u + g * D;
      const float* k = u + (G + g) * D;
      float sq = 0.f, sk = 0.f, dot = 0.f;
      for (int i = lane; i < D; i += 64) {
        sq += q[i] * q[i];
        sk += k[i] * k[i];
        dot += q[i] * k[i];
      }
      const float rq = a.qscale / sqrtf(wave_sum(sq) + 1e-6f), rk = 1.f / sqrtf(wave_sum(sk) + 1e-6f);
      dot = wave_sum(dot);
      float* qo = a.qk + (t * 2 * G + g) * a.Dp;
      float* ko = a.qk + ((t * 2 + 1) * G + g) * a.Dp;
      for (int i = lane; i < a.Dp; i += 64) {
        qo[i] = i < D ? q[i] * rq : 0.f;
        ko[i] = i < D ? k[i] * rk : 0.f;
      }
      if (lane == 0) a.kq[t * G + g] = dot * rq * rk;
    }
    const float* v = u + 2 * G * D;
    float* vo = a.v + t * H * a.Dvp;
    if (a.Dvp == Dv) {
      for (int i = threadIdx.x; i < H * Dv; i += 256) vo[i] = v[i];
    } else {
      for (int i = threadIdx.x; i < H * a.Dvp; i += 256) {
        const int h = i / a.Dvp, c = i - h * a.Dvp;
        vo[i] = c < Dv ? v[h * Dv + c] : 0.f;
      }
    }
    if (rr + 1 < count) __syncthreads();             // the next row reuses the buffer
  }
  if (hist > 0 && st != nullptr && t0 == s.first) {
    __syncthreads();                                 // every thread has read the old inputs
    conv_keep(a.in, s, st);
  }
}

// What the two forms of the recurrence share.
struct DeltaArgs {
  const float* qk;
  const float* v;
  const float2* gates;
  const float* kq;
  float* state;                  // [slots, stride]: per head S [D, Dv]
  long long state_stride;
  const int32_t* cu_q;
  const int32_t* positions;
  const int32_t* slots;
  float* out;                    // [T, H * Dv]
  int H, G, D, Dp, Dv, Dvp;
  int short_rows;                // portions of up to this many rows run row by row, longer ones in chunks
  // chunks of all portions, compactly: chunk c of sequence b has index cu_q[b] / 64 + b + c
  float* w;                      // [chunks, H, 64, Dp]
  float* kt;                     // [chunks, H, Dp, 64]   (e^(L_last - L_t) k_t)^T, zero past the portion's end
  float* ut;                     // [chunks, H, Dvp, 64]  (T diag(beta) V)^T
  float* u;                      // [chunks, H, Dvp, 64]  U^T
  float* s0;                     // [chunks, H, Dvp, Dp]  state at the chunk's start, transposed
  double* cum;                   // [chunks, H, 64]       cumulative log decays L
  float* decay;                  // [chunks, H]           e^(L_last)
};

// ---------------------------------------------------------------- row by row
// One block of four waves per (64 value columns, head, sequence). Lane = column, wave w keeps rows w * DR .. of the state
// column in registers. S^T k and S^T q of the decayed state come from one pass over it (o = g S^T q + (k . q) u), the four
// waves' parts through LDS.
template <int DR>
__global__ __launch_bounds__(256) void delta_scan_kernel(DeltaArgs a) {
  __shared__ float qs[4 * DR], ks[4 * DR];
  __shared__ float part[2][4][64];
  const int b = blockIdx.z, h = blockIdx.y, g = h / (a.H / a.G);
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int dv = blockIdx.x * 64 + lane;
  const int slot = a.slots[b];
  const int q0 = a.cu_q[b], q1 = a.cu_q[b + 1];
  if (slot < 0 || q1 <= q0 || q1 - q0 > a.short_rows) return;         // the same for the whole block
  const bool live = dv < a.Dv;
  const int d0 = wave * DR;
  float* st = a.state + static_cast<size_t>(slot) * a.state_stride + static_cast<size_t>(h) * a.D * a.Dv;
  const bool fresh = a.positions[q0] == 0;
  float S[DR];
#pragma unroll
  for (int i = 0; i < DR; ++i) S[i] = !fresh && live && d0 + i < a.D ? st[static_cast<size_t>(d0 + i) * a.Dv + dv] : 0.f;
  for (int t = q0; t < q1; ++t) {
    for (int i = threadIdx.x; i < 4 * DR; i += 256) {
      const bool in = i < a.Dp;
      qs[i] = in ? a.qk[(static_cast<size_t>(t) * 2 * a.G + g) * a.Dp + i] : 0.f;
      ks[i] = in ? a.qk[((static_cast<size_t>(t) * 2 + 1) * a.G + g) * a.Dp + i] : 0.f;
    }
    const float2 gate = a.gates[static_cast<size_t>(t) * a.H + h];
    const float decay = expf(gate.y);
    const float vv = live ? a.v[(static_cast<size_t>(t) * a.H + h) * a.Dvp + dv] : 0.f;
    const float kq = a.kq[static_cast<size_t>(t) * a.G + g];
    __syncthreads();
    float pk = 0.f, pq = 0.f;
#pragma unroll
    for (int i = 0; i < DR; ++i) {
      S[i] *= decay;
      pk += S[i] * ks[d0 + i];
      pq += S[i] * qs[d0 + i];
    }
    part[0][wave][lane] = pk;
    part[1][wave][lane] = pq;
    __syncthreads();
    pk = part[0][0][lane] + part[0][1][lane] + part[0][2][lane] + part[0][3][lane];
    pq = part[1][0][lane] + part[1][1][lane] + part[1][2][lane] + part[1][3][lane];
    const float u = gate.x * (vv - pk);
#pragma unroll
    for (int i = 0; i < DR; ++i) S[i] += ks[d0 + i] * u;
    if (wave == 0 && live) a.out[static_cast<size_t>(t) * a.H * a.Dv + h * a.Dv + dv] = pq + kq * u;
    if (t + 1 < q1) __syncthreads();                 // the operands and the parts are replaced
  }
  if (live) {
#pragma unroll
    for (int i = 0; i < DR; ++i)
      if (d0 + i < a.D) st[static_cast<size_t>(d0 + i) * a.Dv + dv] = S[i];
  }
}

// ---------------------------------------------------------------- chunks of 64 rows
// With L_t the sum of the log decays of the chunk's rows up to t and S0 the state at its start, unrolling the rule gives
//   S_t = e^(L_t) S0 + sum_(r <= t) e^(L_t - L_r) k_r u_r^T,
//   u_t + beta_t sum_(r < t) e^(L_t - L_r) (k_r . k_t) u_r = beta_t (v_t - e^(L_t) S0^T k_t),
// i.e. (I + A) U = diag(beta) V - diag(beta e^L) K S0 with A strictly lower triangular. With T = (I + A)^-1 (its entries stay
// below one in size, as the rule only ever shrinks what it reads at a unit key):
//   1. delta_chunk_kernel: per (chunk, head), all side by side: A, T by 16 x 16 blocks, W = T diag(beta e^L) K and
//      T diag(beta) V;
//   2. delta_state_kernel: per (16 value columns, head, sequence), chunk after chunk: U = T diag(beta) V - W S0, then
//      S0 <- e^(L_last) S0 + sum_r e^(L_last - L_r) k_r u_r^T; leaves U and every chunk's S0;
//   3. delta_out_kernel: per (chunk, head), side by side: o_t = e^(L_t) S0^T q_t + sum_(r <= t) e^(L_t - L_r) (q_t . k_r) u_r.
// All products run on v_mfma_f32_16x16x4_f32. An operand's four depth indices of one MFMA are 16 kk + 4 (lane >> 4) + i for
// i = 0..3 (which indices meet is free as long as both operands agree), so operands that are contiguous in the depth are read
// 16 bytes at a time. Rows past the portion's end have beta 0 and log decay 0: they change nothing.
constexpr int kChunk = 64;
constexpr int kTS = kChunk + 4;                      // row stride of 64 x 64 matrices in LDS

LC_DEVICE f32x4 mfma4(const float4& x, const float4& y, f32x4 acc) {
  acc = __builtin_amdgcn_mfma_f32_16x16x4f32(x.x, y.x, acc, 0, 0, 0);
  acc = __builtin_amdgcn_mfma_f32_16x16x4f32(x.y, y.y, acc, 0, 0, 0);
  acc = __builtin_amdgcn_mfma_f32_16x16x4f32(x.z, y.z, acc, 0, 0, 0);
  return __builtin_amdgcn_mfma_f32_16x16x4f32(x.w, y.w, acc, 0, 0, 0);
}

LC_DEVICE float4 lds4(const float* p) { return *reinterpret_cast<const float4*>(p); }

// Rows of chunk c of sequence b: first row, how many (0: none or not in chunks), index among all chunks.
struct Chunk {
  int row0, rows;
  size_t index;
};
LC_DEVICE Chunk chunk_of(const DeltaArgs& a, int b, int c) {
  const int q0 = a.cu_q[b], q1 = a.cu_q[b + 1];
  Chunk k{q0 + c * kChunk, 0, static_cast<size_t>(q0 / kChunk + b + c)};
  if (a.slots[b] >= 0 && q1 - q0 > a.short_rows) k.rows = max(0, min(kChunk, q1 - k.row0));
  return k;
}

__global__ __launch_bounds__(256) void delta_chunk_kernel(DeltaArgs a) {
  extern __shared__ float lds[];
  __shared__ double cum[kChunk];
  __shared__ float beta[kChunk], bdec[kChunk];       // beta, beta e^L
  __shared__ float rest[kChunk];                     // e^(L_last - L), zero past the portion's end
  const int h = blockIdx.y, g = h / (a.H / a.G);
  const Chunk ck = chunk_of(a, blockIdx.z, blockIdx.x);
  if (ck.rows == 0) return;                          // the same for the whole block
  const int Dp = a.Dp, DS = Dp + 4;
  float* Ks = lds;                                   // [64][DS]
  float* Ts = Ks + kChunk * DS;                      // [64][kTS]: A, then T in place, block row after block row
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, lr = lane & 15, lk = lane >> 4;
  const int last = ck.row0 + ck.rows - 1;
  for (int i = threadIdx.x; i < kChunk * (Dp / 4); i += 256) {
    const int r = i / (Dp / 4), c = i - r * (Dp / 4);
    const size_t row = min(ck.row0 + r, last);
    *reinterpret_cast<float4*>(Ks + r * DS + 4 * c) = reinterpret_cast<const float4*>(a.qk + ((row * 2 + 1) * a.G + g) * Dp)[c];
  }
  if (wave == 0) {
    const bool in = lane < ck.rows;
    const float2 gate = in ? a.gates[static_cast<size_t>(ck.row0 + lane) * a.H + h] : make_float2(0.f, 0.f);
    double L = gate.y;
#pragma unroll
    for (int off = 1; off < 64; off <<= 1) {
      const double p = __shfl_up(L, off, 64);
      if (lane >= off) L += p;
    }
    cum[lane] = L;
    beta[lane] = gate.x;
    bdec[lane] = gate.x * expf(static_cast<float>(L));
    a.cum[(ck.index * a.H + h) * kChunk + lane] = L;
    const double end = __shfl(L, 63, 64);
    rest[lane] = in ? expf(static_cast<float>(end - L)) : 0.f;
    if (lane == 0) a.decay[ck.index * a.H + h] = expf(static_cast<float>(end));
  }
  __syncthreads();
  float* kt = a.kt + (ck.index * a.H + h) * Dp * kChunk;
  for (int i = threadIdx.x; i < Dp * (kChunk / 4); i += 256) {       // neighbouring lanes: neighbouring keys' coordinates
    const int d = i % Dp, t = 4 * (i / Dp);
    const float* k = Ks + t * DS + d;
    *reinterpret_cast<float4*>(kt + d * kChunk + t) = make_float4(k[0] * rest[t], k[DS] * rest[t + 1], k[2 * DS] * rest[t + 2], k[3 * DS] * rest[t + 3]);
  }
  for (int ct = 0; ct <= wave; ++ct) {               // wave w: rows 16 w .. 16 w + 15 of A
    f32x4 s0 = {0.f, 0.f, 0.f, 0.f}, s1 = {0.f, 0.f, 0.f, 0.f};
    for (int kk = 0; kk < Dp; kk += 16) {
      const float4 x = lds4(Ks + (16 * wave + lr) * DS + kk + 4 * lk), y = lds4(Ks + (16 * ct + lr) * DS + kk + 4 * lk);
      s0 = __builtin_amdgcn_mfma_f32_16x16x4f32(x.x, y.x, s0, 0, 0, 0);
      s1 = __builtin_amdgcn_mfma_f32_16x16x4f32(x.y, y.y, s1, 0, 0, 0);
      s0 = __builtin_amdgcn_mfma_f32_16x16x4f32(x.z, y.z, s0, 0, 0, 0);
      s1 = __builtin_amdgcn_mfma_f32_16x16x4f32(x.w, y.w, s1, 0, 0, 0);
    }
    const int r = 16 * ct + lr;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int t = 16 * wave + 4 * lk + i;
      Ts[t * kTS + r] = r < t ? beta[t] * expf(static_cast<float>(cum[t] - cum[r])) * (s0[i] + s1[i]) : 0.f;
    }
  }
  __syncthreads();
  {                                                  // diagonal blocks: wave w inverts block w, a lane per column
    float x[16];
    const float* Aw = Ts + 16 * wave * kTS + 16 * wave;
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      float v = i == lr ? 1.f : 0.f;
#pragma unroll
      for (int m = 0; m < i; ++m) v -= Aw[i * kTS + m] * x[m];
      x[i] = v;
    }
    __syncthreads();                                 // (every lane has read its block)
    if (lk == 0) {
#pragma unroll
      for (int i = 0; i < 16; ++i) Ts[(16 * wave + i) * kTS + 16 * wave + lr] = x[i];
    }
  }
  __syncthreads();
  // block row i: T_ij = -T_ii sum_(j <= k < i) A_ik T_kj. A product's accumulator is the next product's right operand as it
  // is (depth index 4 (lane >> 4) + i in register i).
  for (int i = 1; i < 4; ++i) {
    f32x4 tij = {0.f, 0.f, 0.f, 0.f};
    if (wave < i) {
      f32x4 m = {0.f, 0.f, 0.f, 0.f};
      for (int k = wave; k < i; ++k) {
        const float* col = Ts + (16 * k + 4 * lk) * kTS + 16 * wave + lr;
        m = mfma4(lds4(Ts + (16 * i + lr) * kTS + 16 * k + 4 * lk), make_float4(col[0], col[kTS], col[2 * kTS], col[3 * kTS]), m);
      }
      tij = mfma4(lds4(Ts + (16 * i + lr) * kTS + 16 * i + 4 * lk), make_float4(-m[0], -m[1], -m[2], -m[3]), tij);
    }
    __syncthreads();                                 // block row i of A has been read
    if (wave < i) {
#pragma unroll
      for (int e = 0; e < 4; ++e) Ts[(16 * i + 4 * lk + e) * kTS + 16 * wave + lr] = tij[e];
    }
    __syncthreads();
  }
  float4 T[10];                                      // lower block triangle, row i from i (i + 1) / 2 on
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int k = 0; k <= i; ++k) T[i * (i + 1) / 2 + k] = lds4(Ts + (16 * i + lr) * kTS + 16 * k + 4 * lk);
  const int nd = Dp / 16, nv = a.Dvp / 16;
  float* wo = a.w + (ck.index * a.H + h) * kChunk * Dp;
  float* uo = a.ut + (ck.index * a.H + h) * a.Dvp * kChunk;
  for (int ct = wave; ct < nd + nv; ct += 4) {       // 16 columns of K or V
    const bool key = ct < nd;
    const int col = key ? 16 * ct + lr : 16 * (ct - nd) + lr;
    float4 B[4];
#pragma unroll
    for (int k = 0; k < 4; ++k) {
      const int r = 16 * k + 4 * lk;
      float e[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        if (key) e[i] = Ks[(r + i) * DS + col] * bdec[r + i];
        else e[i] = a.v[(static_cast<size_t>(min(ck.row0 + r + i, last)) * a.H + h) * a.Dvp + col] * beta[r + i];
      }
      B[k] = make_float4(e[0], e[1], e[2], e[3]);
    }
    f32x4 acc[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) acc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int k = 0; k < 4; ++k)
#pragma unroll
      for (int i = k; i < 4; ++i) acc[i] = mfma4(T[i * (i + 1) / 2 + k], B[k], acc[i]);
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      if (key) {
#pragma unroll
        for (int e = 0; e < 4; ++e) wo[(16 * i + 4 * lk + e) * Dp + col] = acc[i][e];
      } else {
        *reinterpret_cast<float4*>(uo + static_cast<size_t>(col) * kChunk + 16 * i + 4 * lk) = make_float4(acc[i][0], acc[i][1], acc[i][2], acc[i][3]);
      }
    }
  }
}

// Pass 2. A block keeps 16 columns of the state: in accumulators (wave w: its 16-row tiles w, w + 4, ...) and, as the right
// operand of U, transposed in LDS. The loop over chunks is one dependent chain, so its body has no branches and the next
// chunk's operands are loaded (ahead of the stores, which then need not be waited for) while the current one is computed.
// DT: 16-row tiles of the key width (Dp = 16 DT).
template <int DT>
struct DeltaChunkRegs {
  float4 w[DT];                                      // rows 16 wave + lr of W
  float4 k[(DT + 3) / 4][4];                         // rows of (e^(L_last - L_t) k_t)^T
  float4 uv;
  float all;                                         // e^(L_last)
};

template <int DT>
__global__ __launch_bounds__(256) void delta_state_kernel(DeltaArgs a) {
  constexpr int NT = (DT + 3) / 4, Dp = 16 * DT;
  __shared__ __attribute__((aligned(16))) float Ss[16][Dp + 4];
  __shared__ __attribute__((aligned(16))) float Us[16][kTS];
  const int h = blockIdx.x, b = blockIdx.z;          // (a head's blocks on one chiplet: they read the same W and K)
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, lr = lane & 15, lk = lane >> 4;
  const int col = blockIdx.y * 16 + lr;
  const int q0 = a.cu_q[b], q1 = a.cu_q[b + 1];
  const int slot = a.slots[b];
  if (slot < 0 || q1 - q0 <= a.short_rows) return;
  const int chunks = (q1 - q0 + kChunk - 1) / kChunk;
  float* st = a.state + static_cast<size_t>(slot) * a.state_stride + static_cast<size_t>(h) * a.D * a.Dv;
  const bool fresh = a.positions[q0] == 0;
  auto mine = [&](int n) { return DT % 4 == 0 || wave + 4 * n < DT; };       // whether the wave has an n-th tile
  f32x4 S[NT];
#pragma unroll
  for (int n = 0; n < NT; ++n)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int d = 16 * (wave + 4 * n) + 4 * lk + e;
      S[n][e] = !fresh && d < a.D && col < a.Dv ? st[static_cast<size_t>(d) * a.Dv + col] : 0.f;
    }
  const size_t first = chunk_of(a, b, 0).index;
  const int w_at = (16 * wave + lr) * Dp + 4 * lk, u_at = col * kChunk + 16 * wave + 4 * lk;
  auto fetch = [&](int c, DeltaChunkRegs<DT>& r) {
    const size_t ch = (first + c) * a.H + h;
    const float* w = a.w + ch * kChunk * Dp + w_at;
    const float* k = a.kt + ch * Dp * kChunk + (16 * wave + lr) * kChunk + 4 * lk;
#pragma unroll
    for (int kk = 0; kk < DT; ++kk) r.w[kk] = lds4(w + 16 * kk);
    r.uv = lds4(a.ut + ch * a.Dvp * kChunk + u_at);
#pragma unroll
    for (int n = 0; n < NT; ++n)
      if (mine(n)) {
#pragma unroll
        for (int kk = 0; kk < 4; ++kk) r.k[n][kk] = lds4(k + 4 * n * 16 * kChunk + 16 * kk);
      }
    r.all = a.decay[ch];
  };
  auto step = [&](int c, const DeltaChunkRegs<DT>& cur, DeltaChunkRegs<DT>& nxt) {
    const size_t ch = (first + c) * a.H + h;
#pragma unroll
    for (int n = 0; n < NT; ++n)
      if (mine(n)) *reinterpret_cast<float4*>(&Ss[lr][16 * (wave + 4 * n) + 4 * lk]) = make_float4(S[n][0], S[n][1], S[n][2], S[n][3]);
    __syncthreads();
    fetch(min(c + 1, chunks - 1), nxt);
    __builtin_amdgcn_sched_barrier(0);               // (the loads are issued here, not where their first use is near)
    float* s0 = a.s0 + (ch * a.Dvp + col) * Dp + 4 * lk;
#pragma unroll
    for (int n = 0; n < NT; ++n)
      if (mine(n)) *reinterpret_cast<float4*>(s0 + 16 * (wave + 4 * n)) = make_float4(S[n][0], S[n][1], S[n][2], S[n][3]);
    f32x4 u0 = {0.f, 0.f, 0.f, 0.f}, u1 = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int kk = 0; kk < DT; ++kk) {
      const float4 y = lds4(&Ss[lr][16 * kk + 4 * lk]);
      u0 = __builtin_amdgcn_mfma_f32_16x16x4f32(cur.w[kk].x, y.x, u0, 0, 0, 0);
      u1 = __builtin_amdgcn_mfma_f32_16x16x4f32(cur.w[kk].y, y.y, u1, 0, 0, 0);
      u0 = __builtin_amdgcn_mfma_f32_16x16x4f32(cur.w[kk].z, y.z, u0, 0, 0, 0);
      u1 = __builtin_amdgcn_mfma_f32_16x16x4f32(cur.w[kk].w, y.w, u1, 0, 0, 0);
    }
    const float4 u = make_float4(cur.uv.x - u0[0] - u1[0], cur.uv.y - u0[1] - u1[1], cur.uv.z - u0[2] - u1[2], cur.uv.w - u0[3] - u1[3]);
    *reinterpret_cast<float4*>(&Us[lr][16 * wave + 4 * lk]) = u;
    *reinterpret_cast<float4*>(a.u + ch * a.Dvp * kChunk + u_at) = u;
    __syncthreads();
    float4 y[4];
#pragma unroll
    for (int kk = 0; kk < 4; ++kk) y[kk] = lds4(&Us[lr][16 * kk + 4 * lk]);
#pragma unroll
    for (int n = 0; n < NT; ++n)
#pragma unroll
      for (int e = 0; e < 4; ++e) S[n][e] *= cur.all;
#pragma unroll
    for (int kk = 0; kk < 4; ++kk)
#pragma unroll
      for (int n = 0; n < NT; ++n)
        if (mine(n)) S[n] = mfma4(cur.k[n][kk], y[kk], S[n]);
  };
  DeltaChunkRegs<DT> even, odd;                      // two sets in turn: nothing is moved between them
  fetch(0, even);
  for (int c = 0; c < chunks; c += 2) {
    step(c, even, odd);
    if (c + 1 < chunks) step(c + 1, odd, even);
  }
#pragma unroll
  for (int n = 0; n < NT; ++n)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int d = 16 * (wave + 4 * n) + 4 * lk + e;
      if (d < a.D && col < a.Dv) st[static_cast<size_t>(d) * a.Dv + col] = S[n][e];
    }
}

// Pass 3. blockIdx.y: head and group of 128 value columns; a wave owns two tiles of 16 columns and all 64 rows.
constexpr int kOutCols = 128;

__global__ __launch_bounds__(256) void delta_out_kernel(DeltaArgs a) {
  extern __shared__ float lds[];
  __shared__ double cum[kChunk];
  const int groups = (a.Dvp + kOutCols - 1) / kOutCols;
  const int h = blockIdx.y / groups, cg = blockIdx.y % groups, g = h / (a.H / a.G);
  const Chunk ck = chunk_of(a, blockIdx.z, blockIdx.x);
  if (ck.rows == 0) return;                          // the same for the whole block
  const int Dp = a.Dp, DS = Dp + 4, nd = Dp / 16;
  float* Qs = lds;                                   // [64][DS]
  float* Ps = Qs + kChunk * DS;                      // [64][kTS]: e^(L_t - L_r) (q_t . k_r), r <= t
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, lr = lane & 15, lk = lane >> 4;
  const int last = ck.row0 + ck.rows - 1;
  const size_t ch = ck.index * a.H + h;
  for (int i = threadIdx.x; i < kChunk * (Dp / 4); i += 256) {
    const int r = i / (Dp / 4), c = i - r * (Dp / 4);
    const size_t row = min(ck.row0 + r, last);
    *reinterpret_cast<float4*>(Qs + r * DS + 4 * c) = reinterpret_cast<const float4*>(a.qk + (row * 2 * a.G + g) * Dp)[c];
  }
  if (threadIdx.x < kChunk) cum[threadIdx.x] = a.cum[ch * kChunk + threadIdx.x];
  __syncthreads();
  for (int ct = 0; ct <= wave; ++ct) {
    const size_t krow = min(ck.row0 + 16 * ct + lr, last);
    const float* k = a.qk + ((krow * 2 + 1) * a.G + g) * Dp + 4 * lk;
    f32x4 s = {0.f, 0.f, 0.f, 0.f};
    for (int kk = 0; kk < Dp; kk += 16)
      s = mfma4(lds4(Qs + (16 * wave + lr) * DS + kk + 4 * lk), *reinterpret_cast<const float4*>(k + kk), s);
    const int r = 16 * ct + lr;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int t = 16 * wave + 4 * lk + i;
      Ps[t * kTS + r] = r <= t ? expf(static_cast<float>(cum[t] - cum[r])) * s[i] : 0.f;
    }
  }
  __syncthreads();
  const int tile = (cg * kOutCols) / 16 + 2 * wave;  // first of the wave's two column tiles
  const int ntile = min(2, a.Dvp / 16 - tile);
  if (ntile <= 0) return;                            // (no barrier follows)
  f32x4 acc[2][4];
#pragma unroll
  for (int n = 0; n < 2; ++n)
#pragma unroll
    for (int i = 0; i < 4; ++i) acc[n][i] = f32x4{0.f, 0.f, 0.f, 0.f};
  const int c0 = 16 * tile + lr, c1 = 16 * (tile + (ntile > 1 ? 1 : 0)) + lr;      // (a single tile is computed twice)
  const float* s0 = a.s0 + (ch * a.Dvp + c0) * Dp + 4 * lk;
  const float* s1 = a.s0 + (ch * a.Dvp + c1) * Dp + 4 * lk;
  float4 b0 = *reinterpret_cast<const float4*>(s0), b1 = *reinterpret_cast<const float4*>(s1);
  for (int kk = 0; kk < nd; ++kk) {
    const float4 x0 = b0, x1 = b1;
    if (kk + 1 < nd) {
      b0 = *reinterpret_cast<const float4*>(s0 + 16 * (kk + 1));
      b1 = *reinterpret_cast<const float4*>(s1 + 16 * (kk + 1));
    }
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const float4 q = lds4(Qs + (16 * i + lr) * DS + 16 * kk + 4 * lk);
      acc[0][i] = mfma4(q, x0, acc[0][i]);
      acc[1][i] = mfma4(q, x1, acc[1][i]);
    }
  }
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const float dec = expf(static_cast<float>(cum[16 * i + 4 * lk + e]));
      acc[0][i][e] *= dec;
      acc[1][i][e] *= dec;
    }
  const float* u0 = a.u + (ch * a.Dvp + c0) * kChunk + 4 * lk;
  const float* u1 = a.u + (ch * a.Dvp + c1) * kChunk + 4 * lk;
#pragma unroll
  for (int k = 0; k < 4; ++k) {
    const float4 x0 = *reinterpret_cast<const float4*>(u0 + 16 * k), x1 = *reinterpret_cast<const float4*>(u1 + 16 * k);
#pragma unroll
    for (int i = k; i < 4; ++i) {
      const float4 p = lds4(Ps + (16 * i + lr) * kTS + 16 * k + 4 * lk);
      acc[0][i] = mfma4(p, x0, acc[0][i]);
      acc[1][i] = mfma4(p, x1, acc[1][i]);
    }
  }
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int t = 16 * i + 4 * lk + e;
      if (t >= ck.rows) continue;
      float* o = a.out + static_cast<size_t>(ck.row0 + t) * a.H * a.Dv + h * a.Dv;
      if (c0 < a.Dv) o[c0] = acc[0][i][e];
      if (ntile > 1 && c1 < a.Dv) o[c1] = acc[1][i][e];
    }
}

// ---------------------------------------------------------------- differential attention: two maps of a head
// o [T, G, 2, H / G, Dv] (map results: key/value head, map, head of the group) -> per head
// y = o_1 - lambda o_2, y / sqrt(mean(y^2) + eps) * scale, head after head into ``out`` (row stride ldo, activation type).
// A wave per (row, head).
template <bool AF32>
__global__ __launch_bounds__(256) void diff_norm_kernel(const float* __restrict__ o, float lambda, float eps, float scale,
                                                        void* __restrict__ out, int ldo, int T, int H, int G, int Dv) {
  const long long idx = static_cast<long long>(blockIdx.x) * 4 + (threadIdx.x >> 6);
  const int lane = threadIdx.x & 63;
  if (idx >= static_cast<long long>(T) * H) return;
  const size_t t = idx / H;
  const int h = static_cast<int>(idx % H), rep = H / G;
  const float* o1 = o + ((t * G + h / rep) * 2 * rep + h % rep) * Dv;
  const float* o2 = o1 + static_cast<size_t>(rep) * Dv;
  float ss = 0.f;
  float y[8];
#pragma unroll
  for (int i = 0; i < 8; ++i) {                       // value heads of up to 512 columns
    const int c = lane + 64 * i;
    y[i] = c < Dv ? o1[c] - lambda * o2[c] : 0.f;
    ss += y[i] * y[i];
  }
  const float r = scale / sqrtf(wave_sum(ss) / static_cast<float>(Dv) + eps);
#pragma unroll
  for (int i = 0; i < 8; ++i) {
    const int c = lane + 64 * i;
    if (c < Dv) Act<AF32>::store(static_cast<typename Act<AF32>::type*>(out), t * ldo + static_cast<size_t>(h) * Dv + c, y[i] * r);
  }
}

int round16(int n) { return (n + 15) / 16 * 16; }

// Padded key width: the state pass is compiled for these numbers of 16-coordinate tiles.
int pad_keys(int d) {
  for (int t : {1, 2, 3, 4, 6, 8, 12, 16})
    if (d <= 16 * t) return 16 * t;
  return round16(d);
}

constexpr int kShortRows = 16;                       // portions of up to this many rows run row by row

size_t chunk_slots(int T, int B) { return static_cast<size_t>(T) / kChunk + B + 1; }

}  // namespace

// ================================================================= launchers
LC_EXPORT int lc_delta_prep(const void* proj, int ld, const void* conv_w, int taps, void* state, long long state_stride,
                            int col_b, int col_a, const void* neg_rate, const void* dt_bias, const void* row_seq,
                            const void* cu_q, const void* positions, const void* slots, void* qk, void* v, void* gates,
                            void* kq, int T, int H, int G, int D, int Dv, float qscale, hipStream_t st) {
  if (T <= 0) return 0;
  if (H <= 0 || G <= 0 || H % G || D <= 0 || Dv <= 0 || taps < 1 || conv_w == nullptr) return -1;
  const int C = 2 * G * D + H * Dv;
  if (ld < C || col_b < 0 || col_a < 0 || ld < col_b + H || ld < col_a + H || neg_rate == nullptr || dt_bias == nullptr) return -1;
  if (row_seq == nullptr || cu_q == nullptr || positions == nullptr || slots == nullptr) return -1;
  if (taps > 1 && (state == nullptr || state_stride < static_cast<long long>(taps - 1) * C)) return -1;
  constexpr size_t kMaxLds = 159 * 1024;
  const size_t lds = static_cast<size_t>(C) * sizeof(float);
  if (lds > kMaxLds) return -2;
  static LcDeviceOnce attr_once;
  attr_once.run([&] {
    (void)hipFuncSetAttribute(reinterpret_cast<const void*>(delta_prep_kernel), hipFuncAttributeMaxDynamicSharedMemorySize,
                              static_cast<int>(kMaxLds));
  });
  const ConvIn in{static_cast<const float*>(proj), ld, static_cast<const float*>(conv_w), taps, static_cast<float*>(state),
                  state_stride, C, conv_vec(proj, ld, conv_w, state, state_stride, C)};
  const DeltaPrepArgs a{in, col_b, col_a, static_cast<const float*>(neg_rate), static_cast<const float*>(dt_bias),
                        static_cast<const int32_t*>(row_seq), static_cast<const int32_t*>(cu_q),
                        static_cast<const int32_t*>(positions), static_cast<const int32_t*>(slots), static_cast<float*>(qk),
                        static_cast<float*>(v), static_cast<float2*>(gates), static_cast<float*>(kq), H, G, D, pad_keys(D), Dv,
                        round16(Dv), qscale, T, (T + 7) / 8};
  delta_prep_kernel<<<dim3(8 * ((T + 7) / 8)), dim3(256), lds, st>>>(a);
  LC_RETURN_LAST_ERROR();
}

// Width of the keys and queries that lc_delta_prep writes for heads of D coordinates.
LC_EXPORT long long lc_delta_key_width(int D) { return pad_keys(D); }

// fp32 numbers of scratch for a step of T rows in B sequences, the longest of max_len rows (0: none needed).
LC_EXPORT long long lc_delta_scratch_floats(int T, int B, int max_len, int H, int D, int Dv) {
  if (max_len <= kShortRows) return 0;
  const long long Dp = pad_keys(D), Dvp = round16(Dv);
  return static_cast<long long>(chunk_slots(T, B)) * H * (2 * kChunk * Dp + 2 * Dvp * kChunk + Dvp * Dp + 2 * kChunk + 1);
}

LC_EXPORT int lc_delta_scan(const void* qk, const void* v, const void* gates, const void* kq, void* state,
                            long long state_stride, const void* cu_q, const void* positions, const void* slots, void* out,
                            int T, int B, int H, int G, int D, int Dv, int max_len, void* scratch, hipStream_t st) {
  if (B <= 0 || T <= 0) return 0;
  if (H <= 0 || G <= 0 || H % G || D <= 0 || Dv <= 0 || D > 256 || state_stride < static_cast<long long>(H) * D * Dv) return -1;
  const int Dp = pad_keys(D), Dvp = round16(Dv);
  const bool chunked = max_len > kShortRows;
  if (chunked && scratch == nullptr) return -1;
  DeltaArgs a{static_cast<const float*>(qk), static_cast<const float*>(v), static_cast<const float2*>(gates),
              static_cast<const float*>(kq), static_cast<float*>(state), state_stride, static_cast<const int32_t*>(cu_q),
              static_cast<const int32_t*>(positions), static_cast<const int32_t*>(slots), static_cast<float*>(out), H, G, D, Dp,
              Dv, Dvp, kShortRows, nullptr, nullptr, nullptr, nullptr, nullptr, nullptr, nullptr};
  if (chunked) {
    const size_t n = chunk_slots(T, B) * H;
    a.cum = static_cast<double*>(scratch);           // (the widest type first)
    a.w = reinterpret_cast<float*>(a.cum + n * kChunk);
    a.kt = a.w + n * kChunk * Dp;
    a.ut = a.kt + n * kChunk * Dp;
    a.u = a.ut + n * Dvp * kChunk;
    a.s0 = a.u + n * Dvp * kChunk;
    a.decay = a.s0 + n * Dvp * Dp;
    const int nc = (max_len + kChunk - 1) / kChunk;
    const int groups = (Dvp + kOutCols - 1) / kOutCols;
    const size_t lds = static_cast<size_t>(kChunk) * (Dp + 4 + kTS) * sizeof(float);
    static LcDeviceOnce attr_once;
    attr_once.run([&] {
      const int most = kChunk * (256 + 4 + kTS) * static_cast<int>(sizeof(float));
      (void)hipFuncSetAttribute(reinterpret_cast<const void*>(delta_chunk_kernel), hipFuncAttributeMaxDynamicSharedMemorySize, most);
      (void)hipFuncSetAttribute(reinterpret_cast<const void*>(delta_out_kernel), hipFuncAttributeMaxDynamicSharedMemorySize, most);
    });
    delta_chunk_kernel<<<dim3(nc, H, B), dim3(256), lds, st>>>(a);
    const dim3 sgrid(H, Dvp / 16, B);
    switch (Dp / 16) {
#define LC_DS(DT) case DT: delta_state_kernel<DT><<<sgrid, dim3(256), 0, st>>>(a); break
      LC_DS(1); LC_DS(2); LC_DS(3); LC_DS(4); LC_DS(6); LC_DS(8); LC_DS(12); LC_DS(16);
#undef LC_DS
      default: return -1;
    }
    delta_out_kernel<<<dim3(nc, H * groups, B), dim3(256), lds, st>>>(a);
  }
  if (!chunked || B > 1) {                           // (a lone portion is of one kind)
    const dim3 grid((Dv + 63) / 64, H, B);
    if (D <= 32) delta_scan_kernel<8><<<grid, dim3(256), 0, st>>>(a);
    else if (D <= 64) delta_scan_kernel<16><<<grid, dim3(256), 0, st>>>(a);
    else if (D <= 128) delta_scan_kernel<32><<<grid, dim3(256), 0, st>>>(a);
    else delta_scan_kernel<64><<<grid, dim3(256), 0, st>>>(a);
  }
  LC_RETURN_LAST_ERROR();
}

LC_EXPORT int lc_diff_norm(const void* o, float lambda, float eps, float scale, void* out, int act_f32, int ldo, int T, int H,
                           int G, int Dv, hipStream_t st) {
  if (T <= 0) return 0;
  if (H <= 0 || G <= 0 || H % G || Dv <= 0 || Dv > 512 || ldo < H * Dv) return -1;
  const dim3 grid(static_cast<unsigned>((static_cast<long long>(T) * H + 3) / 4)), block(256);
  if (act_f32) diff_norm_kernel<true><<<grid, block, 0, st>>>(static_cast<const float*>(o), lambda, eps, scale, out, ldo, T, H, G, Dv);
  else diff_norm_kernel<false><<<grid, block, 0, st>>>(static_cast<const float*>(o), lambda, eps, scale, out, ldo, T, H, G, Dv);
  LC_RETURN_LAST_ERROR();
}
