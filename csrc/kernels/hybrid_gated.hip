// Kernels of hybrid decoder designs whose sublayers sit between two norms, gate their result from their own input and
// read the previous token's input beside the current one: the residual step with the gate and both norms in one
// launch, the token shift over per-sequence state, the attention pre-processing with short causal convolutions
// (their last inputs are per-sequence state too), norms over the whole projection or per head, a rotation, a query
// temperature, mixed values and the paged cache write, and the soft cap of the logits.
//
// A step's sequences are described by row_seq [T] (sequence of a row, < 0: padding), cu_q [B + 1] (row ranges),
// positions [T] and slots [B] (state slot of the sequence, < 0: none). A sequence whose first row is at position 0
// starts from zeros, so slots are never cleared. Rows of one launch run in any order: state that a launch both
// reads and replaces is touched only by the block of the sequence's FIRST row, every number by one thread.
#include "hybrid_common.h"

namespace {

// ---------------------------------------------------------------- residual step with a gate and two norms
// With y [T, d] (a product whose depth was split comes as the slabs of its partial sums): v = y * sigmoid(gate) (gate given: logits, row stride ld_gate), then rms-normed times w_out (w_out
// given), x += v. With w_in: h = x / sqrt(mean(x^2) + eps) * w_in, written to ``ha`` in the activation type and, when
// given, to ``h32``. With ``mu`` (steps whose sequences all have ONE row): ``hs`` = h + (h' - h) * mu in the
// activation type, h' the sequence's stored row (zeros at position 0), and h becomes the stored row. With ``w_in2``: ``ha2`` =
// x / sqrt(mean(x^2) + eps) * w_in2 beside it (two sublayers that read the same stream through norms of their own).
// A block per row. Rows of up to 4 * 256 * kStepVec coordinates whose pieces are 16-byte aligned (VEC) stay in registers
// between the sums; others are read again.
constexpr int kStepVec = 4;

LC_DEVICE float4 shift4(const float4& h, const float4& p, const float4& m) {
  return make_float4(h.x + (p.x - h.x) * m.x, h.y + (p.y - h.y) * m.y, h.z + (p.z - h.z) * m.z, h.w + (p.w - h.w) * m.w);
}

struct StepArgs {
  float* x;
  const float* y;                // ``parts`` slabs of [T, d], ``slab`` elements apart, whose sum is the sublayer's result
  int parts;
  size_t slab;
  const float* gate;
  int ld_gate;
  const float* w_out;
  const float* w_in;
  float eps;
  void* ha;
  float* h32;
  const float* w_in2;            // a second norm of the same row (null: none)
  void* ha2;
  // the shift of single-row sequences
  const float* mu;
  float* state;
  long long state_stride;
  const int32_t* row_seq;
  const int32_t* positions;
  const int32_t* slots;
  void* hs;
  int d;
};

template <bool AF32, bool VEC>
__global__ __launch_bounds__(256) void gated_step_kernel(StepArgs a) {
  __shared__ float red[16];
  const int t = blockIdx.x, d = a.d;
  const size_t row = static_cast<size_t>(t) * d;
  const float* grow = a.gate != nullptr ? a.gate + static_cast<size_t>(t) * a.ld_gate : nullptr;
  float* prev = nullptr;                              // the sequence's stored row (null: none)
  bool fresh = true;
  if (a.mu != nullptr) {
    const int b = a.row_seq[t];
    const int slot = b < 0 ? -1 : a.slots[b];
    if (slot >= 0) {
      prev = a.state + static_cast<size_t>(slot) * a.state_stride;
      fresh = a.positions[t] == 0;
    }
  }
  if constexpr (VEC) {
    const int n4 = d / 4;
    float4 xv[kStepVec], yv[kStepVec];
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < kStepVec; ++i) {
      const int c = threadIdx.x + 256 * i;
      xv[i] = yv[i] = make_float4(0.f, 0.f, 0.f, 0.f);
      if (c < n4) {
        xv[i] = reinterpret_cast<const float4*>(a.x + row)[c];
        if (a.y != nullptr) {
          float4 v = reinterpret_cast<const float4*>(a.y + row)[c];
#pragma unroll 8
          for (int s = 1; s < a.parts; ++s) {       // (several slabs in flight)
            const float4 w = reinterpret_cast<const float4*>(a.y + s * a.slab + row)[c];
            v = make_float4(v.x + w.x, v.y + w.y, v.z + w.z, v.w + w.w);
          }
          if (grow != nullptr) {
            const float4 g = reinterpret_cast<const float4*>(grow)[c];
            v = make_float4(v.x * sigmoidf_(g.x), v.y * sigmoidf_(g.y), v.z * sigmoidf_(g.z), v.w * sigmoidf_(g.w));
          }
          ss += v.x * v.x + v.y * v.y + v.z * v.z + v.w * v.w;
          yv[i] = v;
        }
      }
    }
    if (a.y != nullptr) {
      const float r = a.w_out != nullptr ? 1.f / sqrtf(block_sum(ss, red) / static_cast<float>(d) + a.eps) : 1.f;
#pragma unroll
      for (int i = 0; i < kStepVec; ++i) {
        const int c = threadIdx.x + 256 * i;
        if (c < n4) {
          float4 w = make_float4(1.f, 1.f, 1.f, 1.f);
          if (a.w_out != nullptr) w = reinterpret_cast<const float4*>(a.w_out)[c];
          xv[i].x += yv[i].x * r * w.x;
          xv[i].y += yv[i].y * r * w.y;
          xv[i].z += yv[i].z * r * w.z;
          xv[i].w += yv[i].w * r * w.w;
          reinterpret_cast<float4*>(a.x + row)[c] = xv[i];
        }
      }
    }
    if (a.w_in == nullptr) return;                    // the same for every thread
    float s2 = 0.f;
#pragma unroll
    for (int i = 0; i < kStepVec; ++i) s2 += xv[i].x * xv[i].x + xv[i].y * xv[i].y + xv[i].z * xv[i].z + xv[i].w * xv[i].w;
    const float r2 = 1.f / sqrtf(block_sum(s2, red) / static_cast<float>(d) + a.eps);
#pragma unroll
    for (int i = 0; i < kStepVec; ++i) {
      const int c = threadIdx.x + 256 * i;
      if (c < n4) {
        const float4 w = reinterpret_cast<const float4*>(a.w_in)[c];
        const float4 h = make_float4(xv[i].x * r2 * w.x, xv[i].y * r2 * w.y, xv[i].z * r2 * w.z, xv[i].w * r2 * w.w);
        store_act4<AF32>(a.ha, row + 4 * c, h);
        if (a.w_in2 != nullptr) {
          const float4 w2 = reinterpret_cast<const float4*>(a.w_in2)[c];
          store_act4<AF32>(a.ha2, row + 4 * c, make_float4(xv[i].x * r2 * w2.x, xv[i].y * r2 * w2.y, xv[i].z * r2 * w2.z, xv[i].w * r2 * w2.w));
        }
        if (a.h32 != nullptr) reinterpret_cast<float4*>(a.h32 + row)[c] = h;
        if (a.mu != nullptr) {
          float4 p = make_float4(0.f, 0.f, 0.f, 0.f);
          if (!fresh) p = reinterpret_cast<const float4*>(prev)[c];
          store_act4<AF32>(a.hs, row + 4 * c, shift4(h, p, reinterpret_cast<const float4*>(a.mu)[c]));
          if (prev != nullptr) reinterpret_cast<float4*>(prev)[c] = h;
        }
      }
    }
  } else {
    typedef typename Act<AF32>::type act_t;
    float r = 1.f;
    auto result = [&](int c) {
      float v = a.y[row + c];
      for (int s = 1; s < a.parts; ++s) v += a.y[s * a.slab + row + c];
      return grow != nullptr ? v * sigmoidf_(grow[c]) : v;
    };
    if (a.y != nullptr && a.w_out != nullptr) {
      float ss = 0.f;
      for (int c = threadIdx.x; c < d; c += 256) {
        const float v = result(c);
        ss += v * v;
      }
      r = 1.f / sqrtf(block_sum(ss, red) / static_cast<float>(d) + a.eps);
    }
    float s2 = 0.f;
    for (int c = threadIdx.x; c < d; c += 256) {
      float v = a.x[row + c];
      if (a.y != nullptr) {
        v += result(c) * r * (a.w_out != nullptr ? a.w_out[c] : 1.f);
        a.x[row + c] = v;
      }
      s2 += v * v;
    }
    if (a.w_in == nullptr) return;
    const float r2 = 1.f / sqrtf(block_sum(s2, red) / static_cast<float>(d) + a.eps);
    for (int c = threadIdx.x; c < d; c += 256) {      // (a thread reads what it wrote itself)
      const float h = a.x[row + c] * r2 * a.w_in[c];
      Act<AF32>::store(static_cast<act_t*>(a.ha), row + c, h);
      if (a.w_in2 != nullptr) Act<AF32>::store(static_cast<act_t*>(a.ha2), row + c, a.x[row + c] * r2 * a.w_in2[c]);
      if (a.h32 != nullptr) a.h32[row + c] = h;
      if (a.mu != nullptr) {
        const float p = fresh ? 0.f : prev[c];
        Act<AF32>::store(static_cast<act_t*>(a.hs), row + c, h + (p - h) * a.mu[c]);
        if (prev != nullptr) prev[c] = h;
      }
    }
  }
}

// ---------------------------------------------------------------- token shift
// hs[t] = h[t] + (h' - h[t]) * mu with h' the row before it in the sequence: row t - 1 of the step, or, for the first
// row of a portion, the sequence's stored row (zeros at position 0). The block of the first row then stores the
// portion's last row. One block per row, V = 4 coordinates per thread when the width allows.
template <bool AF32, int V>
__global__ __launch_bounds__(256) void token_shift_kernel(const float* __restrict__ h, const float* __restrict__ mu,
                                                          float* __restrict__ state, long long state_stride,
                                                          const int32_t* __restrict__ row_seq,
                                                          const int32_t* __restrict__ cu_q,
                                                          const int32_t* __restrict__ positions,
                                                          const int32_t* __restrict__ slots, void* __restrict__ hs, int d) {
  const int t = blockIdx.x;
  const RowSeq s = row_sequence(t, row_seq, cu_q, positions, slots);
  const bool first = t == s.first;
  float* st = s.slot >= 0 ? state + static_cast<size_t>(s.slot) * state_stride : nullptr;
  const size_t row = static_cast<size_t>(t) * d;
  const float* last = h + static_cast<size_t>(s.first + s.rows - 1) * d;
  typedef typename Act<AF32>::type act_t;
  for (int c = threadIdx.x * V; c < d; c += 256 * V) {
    if constexpr (V == 4) {
      const float4 v = *reinterpret_cast<const float4*>(h + row + c);
      float4 p = make_float4(0.f, 0.f, 0.f, 0.f);
      if (!first) p = *reinterpret_cast<const float4*>(h + row - d + c);
      else if (!s.fresh) p = *reinterpret_cast<const float4*>(st + c);
      store_act4<AF32>(hs, row + c, shift4(v, p, *reinterpret_cast<const float4*>(mu + c)));
      if (first && st != nullptr) *reinterpret_cast<float4*>(st + c) = *reinterpret_cast<const float4*>(last + c);
    } else {
      const float v = h[row + c];
      const float p = !first ? h[row - d + c] : (s.fresh ? 0.f : st[c]);
      Act<AF32>::store(static_cast<act_t*>(hs), row + c, v + (p - v) * mu[c]);
      if (first && st != nullptr) st[c] = last[c];
    }
  }
}

// ---------------------------------------------------------------- attention pre-processing
// One block per token. qkv [T, ld] fp32: q [H*D] | k [G*D] | v [G*Dv] (C channels in all). In this order, each optional:
//   a causal convolution over time per channel, conv_w [taps, C]: y_t = sum_j w[j] u_(t - taps + 1 + j); inputs before the
//     step come from the sequence's state [taps - 1, C] (oldest first), zeros before the sequence's start. The block
//     of a portion's first row also serves the next taps - 2 rows (they reach into the state as well) and then
//     replaces the state by the portion's last taps - 1 inputs;
//   norm 1: RMS over the whole query (key) projection, weights [H*D] / [G*D]; norm 2: per head, weights [D] shared;
//   rotation of the first rot_dims coordinates of each q and k head (pairs: neighbours, otherwise i with
//     i + rot_dims / 2) by position * inv_freq[i] (angles fp64);
//   temperature: q *= 1 + coef * ln(floor((p + 1) / every) + 1);
//   value mix: v <- (1 - lambda) v + lambda v_first[t]; before it v is written to v_save when given.
// q goes to q_out [T, H*D] fp32, k and v to the paged planes [blocks, G, BS, D] / [blocks, G, BS, Dv]. With ``maps`` > 1 a head
// has several query / key maps over the same values: H and G count the maps of all heads (head by head), GV = G / maps value
// heads; the queries leave in the order (key/value head, map, head of the group), so that those of one key head are neighbours.
struct PrepArgs {
  ConvIn in;                      // q | k | v and their convolution over time
  int norm;
  const float* qn;
  const float* kn;
  float eps;
  const double* inv_freq;
  int rot_dims, pairs;
  float rot_mag;                  // factor on cosine and sine
  float t_coef;                   // 0: no temperature
  double t_every;
  const float* v_first;
  int ld_vf;
  float lambda;
  float* v_save;
  const int32_t* row_seq;
  const int32_t* cu_q;
  const int32_t* positions;
  const int32_t* slots;
  const int32_t* slot_mapping;
  void* kc;
  void* vc;
  float* q_out;
  int H, G, GV, D, Dv, BS;
  int maps;                       // G / GV key heads per value head
  int T, per_xcd;                 // rows, rows per chiplet (neighbouring rows share their inputs, so they share an L2)
};

template <bool CF32>
__global__ __launch_bounds__(256) void attn_prep_kernel(PrepArgs a) {
  extern __shared__ float lds[];
  __shared__ float red[16];
  const int H = a.H, G = a.G, GV = a.GV, D = a.D, Dv = a.Dv;
  const int nq = H * D, nk = G * D, nv = GV * Dv, C = nq + nk + nv;
  float* u = lds;                                    // [C] the token's channels
  float* cs = u + C;                                 // [rot_dims] cos | sin
  const int t0 = (blockIdx.x & 7) * a.per_xcd + (blockIdx.x >> 3);   // (workgroups go round robin over the 8 chiplets)
  if (t0 >= a.T) return;
  const int hist = a.in.taps > 1 ? a.in.taps - 1 : 0;
  RowSeq s{t0, 1, -1, true};
  int count = 1;
  if (hist > 0) {
    s = row_sequence(t0, a.row_seq, a.cu_q, a.positions, a.slots);
    count = conv_rows_of_block(t0, s, hist);
    if (count == 0) return;                          // served by the portion's first row
  }
  float* st = s.slot >= 0 ? a.in.state + static_cast<size_t>(s.slot) * a.in.state_stride : nullptr;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int half = a.rot_dims >> 1;
  for (int rr = 0; rr < count; ++rr) {
    const int t = t0 + rr;
    const int pos = a.positions[t];
    conv_token<false>(a.in, s, st, t - s.first, u);
    for (int j = threadIdx.x; j < half; j += 256) {
      constexpr double kTwoPi = 6.283185307179586476925286766559;
      double ang = static_cast<double>(pos) * a.inv_freq[j];
      ang -= kTwoPi * rint(ang / kTwoPi);
      float sn, cn;
      sincosf(static_cast<float>(ang), &sn, &cn);
      cs[j] = cn * a.rot_mag;
      cs[half + j] = sn * a.rot_mag;
    }
    __syncthreads();
    float temp = 1.f;
    if (a.t_coef != 0.f) temp += a.t_coef * logf(static_cast<float>(floor((pos + 1.0) / a.t_every) + 1.0));
    if (a.norm == 1) {
      float sq = 0.f, sk = 0.f;
      for (int i = threadIdx.x; i < nq; i += 256) sq += u[i] * u[i];
      for (int i = threadIdx.x; i < nk; i += 256) sk += u[nq + i] * u[nq + i];
      const float rq = 1.f / sqrtf(block_sum(sq, red) / static_cast<float>(nq) + a.eps);
      const float rk = 1.f / sqrtf(block_sum(sk, red) / static_cast<float>(nk) + a.eps);
      for (int i = threadIdx.x; i < nq; i += 256) u[i] *= rq * a.qn[i];
      for (int i = threadIdx.x; i < nk; i += 256) u[nq + i] *= rk * a.kn[i];
      __syncthreads();
    } else if (a.norm == 2) {
      for (int g = wave; g < H + G; g += 4) {        // q heads, then key heads: a wave owns a head
        float* head = u + g * D;
        const float* w = g < H ? a.qn : a.kn;
        float ss = 0.f;
        for (int i = lane; i < D; i += 64) ss += head[i] * head[i];
        const float rn = 1.f / sqrtf(wave_sum(ss) / static_cast<float>(D) + a.eps);
        for (int i = lane; i < D; i += 64) head[i] *= rn * w[i];
      }
      __syncthreads();
    }
    auto turned = [&](const float* head, int i) {    // coordinate i of a head
      const float v = head[i];
      if (i >= a.rot_dims) return v;
      if (a.pairs) {
        const float c = cs[i >> 1], sn = cs[half + (i >> 1)], o = head[i ^ 1];
        return (i & 1) ? v * c + o * sn : v * c - o * sn;
      }
      const int j = i < half ? i : i - half;
      const float c = cs[j], sn = cs[half + j];
      return i < half ? v * c - head[i + half] * sn : v * c + head[i - half] * sn;
    };
    const int rep = H / G;
    for (int g = wave; g < H; g += 4) {
      // (several maps per head: the queries of one key head lie side by side)
      const int m = g % a.maps, qh = g / a.maps;
      const int at = ((qh / rep) * a.maps + m) * rep + qh % rep;
      for (int i = lane; i < D; i += 64) a.q_out[static_cast<size_t>(t) * nq + at * D + i] = turned(u + g * D, i) * temp;
    }
    const int slot = a.slot_mapping[t];
    const size_t blk = slot >= 0 ? slot / a.BS : 0, off = slot >= 0 ? slot % a.BS : 0;
    typedef typename Act<CF32>::type cache_t;
    if (slot >= 0)
      for (int g = wave; g < G; g += 4)
        for (int i = lane; i < D; i += 64)
          Act<CF32>::store(static_cast<cache_t*>(a.kc), ((blk * G + g) * a.BS + off) * D + i, turned(u + nq + g * D, i));
    for (int g = wave; g < GV; g += 4)
      for (int i = lane; i < Dv; i += 64) {
        const int at = g * Dv + i;
        float v = u[nq + nk + at];
        if (a.v_save != nullptr) a.v_save[static_cast<size_t>(t) * nv + at] = v;
        if (a.v_first != nullptr) v = (1.f - a.lambda) * v + a.lambda * a.v_first[static_cast<size_t>(t) * a.ld_vf + at];
        if (slot >= 0) Act<CF32>::store(static_cast<cache_t*>(a.vc), ((blk * GV + g) * a.BS + off) * Dv + i, v);
      }
    if (rr + 1 < count) __syncthreads();             // the next row reuses the buffers
  }
  if (hist > 0 && st != nullptr && t0 == s.first) {
    __syncthreads();                                 // every thread has read the old inputs
    conv_keep(a.in, s, st);
  }
}

// ---------------------------------------------------------------- soft cap
// x <- cap * tanh(x / cap), in place.
__global__ void softcap_kernel(float* __restrict__ x, long long n, float cap) {
  const long long i = static_cast<long long>(blockIdx.x) * blockDim.x + threadIdx.x;
  if (i < n) x[i] = cap * tanhf(x[i] / cap);
}

}  // namespace

// ================================================================= launchers
LC_EXPORT int lc_gated_step(void* x, const void* y, int parts, const void* gate, int ld_gate, const void* w_out, const void* w_in,
                            float eps, void* ha, void* h32, const void* w_in2, void* ha2, int act_f32, const void* mu, void* state,
                            long long state_stride, const void* row_seq, const void* positions, const void* slots, void* hs,
                            int T, int d, hipStream_t st) {
  if (T <= 0) return 0;
  if (d <= 0 || parts < 1 || (y == nullptr && w_in == nullptr) || (w_in != nullptr && ha == nullptr)) return -1;
  if (gate != nullptr && (y == nullptr || ld_gate < d)) return -1;
  if (w_in2 != nullptr && (w_in == nullptr || ha2 == nullptr)) return -1;
  if (mu != nullptr && (w_in == nullptr || hs == nullptr || state == nullptr || row_seq == nullptr || positions == nullptr ||
                        slots == nullptr || state_stride < d))
    return -1;
  const StepArgs a{static_cast<float*>(x), static_cast<const float*>(y), parts, static_cast<size_t>(T) * d,
                   static_cast<const float*>(gate), ld_gate, static_cast<const float*>(w_out), static_cast<const float*>(w_in), eps, ha, static_cast<float*>(h32),
                   static_cast<const float*>(w_in2), ha2,
                   static_cast<const float*>(mu), static_cast<float*>(state), state_stride,
                   static_cast<const int32_t*>(row_seq), static_cast<const int32_t*>(positions),
                   static_cast<const int32_t*>(slots), hs, d};
  const bool vec = d % 4 == 0 && d <= 4 * 256 * kStepVec && ld_gate % 4 == 0 && state_stride % 4 == 0 && aligned16(x) &&
                   aligned16(y) && aligned16(gate) && aligned16(w_out) && aligned16(w_in) && aligned16(ha) &&
                   aligned16(h32) && aligned16(w_in2) && aligned16(ha2) && aligned16(mu) && aligned16(state) && aligned16(hs);
#define LC_GS(A32, V) gated_step_kernel<A32, V><<<dim3(T), dim3(256), 0, st>>>(a)
  if (act_f32 && vec) LC_GS(true, true);
  else if (act_f32) LC_GS(true, false);
  else if (vec) LC_GS(false, true);
  else LC_GS(false, false);
#undef LC_GS
  LC_RETURN_LAST_ERROR();
}

LC_EXPORT int lc_token_shift(const void* h, const void* mu, void* state, long long state_stride, const void* row_seq,
                             const void* cu_q, const void* positions, const void* slots, void* hs, int act_f32, int T, int d,
                             hipStream_t st) {
  if (T <= 0) return 0;
  if (d <= 0 || state_stride < d || h == nullptr || mu == nullptr || state == nullptr || slots == nullptr) return -1;
  const bool vec = d % 4 == 0 && state_stride % 4 == 0 && aligned16(h) && aligned16(mu) && aligned16(state) && aligned16(hs);
#define LC_TS(A32, V)                                                                                              \
  token_shift_kernel<A32, V><<<dim3(T), dim3(256), 0, st>>>(                                                       \
      static_cast<const float*>(h), static_cast<const float*>(mu), static_cast<float*>(state), state_stride,       \
      static_cast<const int32_t*>(row_seq), static_cast<const int32_t*>(cu_q), static_cast<const int32_t*>(positions), \
      static_cast<const int32_t*>(slots), hs, d)
  if (act_f32 && vec) LC_TS(true, 4);
  else if (act_f32) LC_TS(true, 1);
  else if (vec) LC_TS(false, 4);
  else LC_TS(false, 1);
#undef LC_TS
  LC_RETURN_LAST_ERROR();
}

LC_EXPORT int lc_attn_prep(const void* qkv, int ld, const void* conv_w, int taps, void* state, long long state_stride,
                           int norm, const void* qn, const void* kn, float eps, const void* inv_freq, int rot_dims, int pairs,
                           float rot_mag, int maps, float t_coef, float t_every, const void* v_first, int ld_vf, float lambda, void* v_save,
                           const void* row_seq, const void* cu_q, const void* positions, const void* slots,
                           const void* slot_mapping, void* kc, void* vc, int cache_f32, void* q_out, int T, int H, int G,
                           int D, int Dv, int BS, hipStream_t st) {
  if (T <= 0) return 0;
  if (H <= 0 || G <= 0 || H % G || D <= 0 || Dv <= 0 || BS <= 0 || kc == nullptr || vc == nullptr || q_out == nullptr) return -1;
  if (maps <= 0 || G % maps) return -1;
  const int GV = G / maps, C = (H + G) * D + GV * Dv;
  if (ld < C || taps < 0 || norm < 0 || norm > 2 || (norm != 0 && (qn == nullptr || kn == nullptr))) return -1;
  if (taps > 0 && conv_w == nullptr) return -1;
  if (taps > 1 && (state == nullptr || state_stride < static_cast<long long>(taps - 1) * C || row_seq == nullptr ||
                   cu_q == nullptr || slots == nullptr))
    return -1;
  if (rot_dims < 0 || rot_dims > D || (rot_dims & 1) || (rot_dims > 0 && inv_freq == nullptr)) return -1;
  if ((t_coef != 0.f && !(t_every > 0.f)) || (v_first != nullptr && ld_vf < GV * Dv)) return -1;
  constexpr size_t kMaxLds = 159 * 1024;             // (the block sums' scratch is static)
  const size_t lds = static_cast<size_t>(C + rot_dims) * sizeof(float);
  if (lds > kMaxLds) return -2;
  static LcDeviceOnce attr_once;
  attr_once.run([&] {
    (void)hipFuncSetAttribute(reinterpret_cast<const void*>(attn_prep_kernel<true>),
                              hipFuncAttributeMaxDynamicSharedMemorySize, static_cast<int>(kMaxLds));
    (void)hipFuncSetAttribute(reinterpret_cast<const void*>(attn_prep_kernel<false>),
                              hipFuncAttributeMaxDynamicSharedMemorySize, static_cast<int>(kMaxLds));
  });
  const ConvIn in{static_cast<const float*>(qkv), ld, static_cast<const float*>(conv_w), taps, static_cast<float*>(state),
                  state_stride, C, conv_vec(qkv, ld, conv_w, state, state_stride, C)};
  const PrepArgs a{in, norm, static_cast<const float*>(qn), static_cast<const float*>(kn), eps,
                   static_cast<const double*>(inv_freq), rot_dims, pairs, rot_mag, t_coef, static_cast<double>(t_every),
                   static_cast<const float*>(v_first), ld_vf, lambda, static_cast<float*>(v_save),
                   static_cast<const int32_t*>(row_seq), static_cast<const int32_t*>(cu_q),
                   static_cast<const int32_t*>(positions), static_cast<const int32_t*>(slots),
                   static_cast<const int32_t*>(slot_mapping), kc, vc, static_cast<float*>(q_out), H, G, GV, D, Dv, BS, maps, T,
                   (T + 7) / 8};
  if (cache_f32) attn_prep_kernel<true><<<dim3(8 * ((T + 7) / 8)), dim3(256), lds, st>>>(a);
  else attn_prep_kernel<false><<<dim3(8 * ((T + 7) / 8)), dim3(256), lds, st>>>(a);
  LC_RETURN_LAST_ERROR();
}

LC_EXPORT int lc_softcap(void* x, long long n, float cap, hipStream_t st) {
  if (n <= 0) return 0;
  if (!(cap > 0.f)) return -1;
  softcap_kernel<<<dim3(static_cast<unsigned>((n + 255) / 256)), dim3(256), 0, st>>>(static_cast<float*>(x), n, cap);
  LC_RETURN_LAST_ERROR();
}
