// Helpers shared by the kernel files of the hybrid decoder designs (hybrid*.hip).
#pragma once
#include "common.h"

namespace {

// An activation-typed buffer (fp32 or bf16, a launch-time flag) read and written as floats.
template <bool F32>
struct Act;
template <>
struct Act<true> {
  typedef float type;
  static LC_DEVICE float load(const float* p, size_t i) { return p[i]; }
  static LC_DEVICE void store(float* p, size_t i, float v) { p[i] = v; }
};
template <>
struct Act<false> {
  typedef bf16_t type;
  static LC_DEVICE float load(const bf16_t* p, size_t i) { return bf16_to_f32(p[i]); }
  static LC_DEVICE void store(bf16_t* p, size_t i, float v) { p[i] = f32_to_bf16(v); }
};

template <bool AF32>
LC_DEVICE void store_act4(void* p, size_t i, const float4& v) {
  if (AF32) {
    *reinterpret_cast<float4*>(static_cast<float*>(p) + i) = v;
  } else {
    *reinterpret_cast<uint2*>(static_cast<bf16_t*>(p) + i) = make_uint2(pack_bf16x2(v.x, v.y), pack_bf16x2(v.z, v.w));
  }
}

// Four neighbouring elements of a table of that type as floats (8- / 16-byte border).
template <bool F32>
LC_DEVICE float4 load_act4(const typename Act<F32>::type* p) {
  if constexpr (F32) {
    return *reinterpret_cast<const float4*>(p);
  } else {
    const uint2 w = *reinterpret_cast<const uint2*>(p);
    return make_float4(__uint_as_float(w.x << 16), __uint_as_float(w.x & 0xffff0000u), __uint_as_float(w.y << 16),
                       __uint_as_float(w.y & 0xffff0000u));
  }
}

LC_DEVICE float sigmoidf_(float x) { return 1.f / (1.f + expf(-x)); }
LC_DEVICE float siluf_(float x) { return x / (1.f + expf(-x)); }
// log sigmoid(z) = min(z, 0) - log1p(exp(-|z|))
LC_DEVICE float logsigmoidf_(float z) { return fminf(z, 0.f) - log1pf(expf(-fabsf(z))); }

// Where a row's sequence starts and which state it owns.
struct RowSeq {
  int first, rows;               // row range of the step
  int slot;                      // < 0: none
  bool fresh;                    // starts at position 0 (or has no state): zeros before it
};

LC_DEVICE RowSeq row_sequence(int t, const int32_t* __restrict__ row_seq, const int32_t* __restrict__ cu_q,
                              const int32_t* __restrict__ positions, const int32_t* __restrict__ slots) {
  RowSeq r{t, 1, -1, true};
  const int b = row_seq[t];
  if (b < 0) return r;
  r.first = cu_q[b];
  r.rows = cu_q[b + 1] - r.first;
  r.slot = slots[b];
  r.fresh = r.slot < 0 || positions[r.first] == 0;
  return r;
}

// ---------------------------------------------------------------- short causal convolution over time
// Per channel y_t = sum_j w[j] u_(t - taps + 1 + j): x [T, ld] the step's inputs (C channels), w [taps, C] (the newest tap
// last); inputs before the step come from the sequence's state [taps - 1, C] (oldest first), zeros before the sequence's
// start. A block of 256 threads serves one token; rows of one launch run in any order, so the block of a portion's first row
// also serves the next taps - 2 rows (they reach into the state as well) and then replaces the state by the portion's last
// taps - 1 inputs.
struct ConvIn {
  const float* x;
  int ld;
  const float* w;
  int taps;                      // 0: the inputs themselves
  float* state;
  long long state_stride;
  int C;
  int vec;                       // every row of x, of the state and of the weights starts on a 16-byte border
};

inline bool aligned16(const void* p) { return reinterpret_cast<uintptr_t>(p) % 16 == 0; }

inline int conv_vec(const void* x, int ld, const void* w, const void* state, long long state_stride, int C) {
  return C % 4 == 0 && ld % 4 == 0 && state_stride % 4 == 0 && aligned16(x) && aligned16(w) && aligned16(state);
}

// Rows that the block of row t0 serves (0: none, the block of the portion's first row does).
LC_DEVICE int conv_rows_of_block(int t0, const RowSeq& s, int hist) {
  const int r = t0 - s.first;
  if (hist <= 0 || r >= hist) return 1;
  return r == 0 ? min(s.rows, hist) : 0;
}

template <bool SILU>
LC_DEVICE float conv_act(float y) { return SILU ? siluf_(y) : y; }

// TAPS input rows (null: zeros), 4 channels per thread and access.
template <int TAPS, bool SILU>
LC_DEVICE void conv_rows4(const ConvIn& a, const RowSeq& s, const float* st, int r, float* u) {
  const float* src[TAPS];
#pragma unroll
  for (int j = 0; j < TAPS; ++j) {
    const int k = r - (TAPS - 1) + j;                // input row inside the portion, < 0: before it
    src[j] = k >= 0 ? a.x + static_cast<size_t>(s.first + k) * a.ld
                    : (s.fresh ? nullptr : st + static_cast<size_t>(k + TAPS - 1) * a.C);
  }
  for (int c = threadIdx.x * 4; c < a.C; c += 1024) {
    float4 x[TAPS], w[TAPS];
#pragma unroll
    for (int j = 0; j < TAPS; ++j) {
      w[j] = *reinterpret_cast<const float4*>(a.w + static_cast<size_t>(j) * a.C + c);
      x[j] = src[j] != nullptr ? *reinterpret_cast<const float4*>(src[j] + c) : make_float4(0.f, 0.f, 0.f, 0.f);
    }
    float4 y = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
    for (int j = 0; j < TAPS; ++j) {
      y.x += w[j].x * x[j].x;
      y.y += w[j].y * x[j].y;
      y.z += w[j].z * x[j].z;
      y.w += w[j].w * x[j].w;
    }
    *reinterpret_cast<float4*>(u + c) = make_float4(conv_act<SILU>(y.x), conv_act<SILU>(y.y), conv_act<SILU>(y.z), conv_act<SILU>(y.w));
  }
}

// u [C] (LDS) = the channels of row r of the portion, convolved, through silu when asked. No barrier.
template <bool SILU>
LC_DEVICE void conv_token(const ConvIn& a, const RowSeq& s, const float* st, int r, float* u) {
  const float* row = a.x + static_cast<size_t>(s.first + r) * a.ld;
  const int hist = a.taps > 1 ? a.taps - 1 : 0;
  if (a.vec && a.taps == 2) {
    conv_rows4<2, SILU>(a, s, st, r, u);
  } else if (a.vec && a.taps == 3) {
    conv_rows4<3, SILU>(a, s, st, r, u);
  } else if (a.vec && a.taps == 4) {
    conv_rows4<4, SILU>(a, s, st, r, u);
  } else if (a.vec && a.taps == 0 && !SILU) {
    for (int c = threadIdx.x * 4; c < a.C; c += 1024) *reinterpret_cast<float4*>(u + c) = *reinterpret_cast<const float4*>(row + c);
  } else if (a.taps > 0) {
    for (int c = threadIdx.x; c < a.C; c += 256) {
      float y = 0.f;
      for (int j = 0; j < a.taps; ++j) {
        const int k = r - hist + j;                  // input row inside the portion, < 0: before it
        float in = 0.f;
        if (k >= 0) in = a.x[static_cast<size_t>(s.first + k) * a.ld + c];
        else if (!s.fresh) in = st[static_cast<size_t>(k + hist) * a.C + c];
        y += a.w[static_cast<size_t>(j) * a.C + c] * in;
      }
      u[c] = conv_act<SILU>(y);
    }
  } else {
    for (int c = threadIdx.x; c < a.C; c += 256) u[c] = conv_act<SILU>(row[c]);
  }
}

// The state becomes the portion's last taps - 1 inputs (by the block of its first row, after every thread of the block
// has read the old ones). A thread owns a channel (four of them): all its inputs are read before one is written.
template <int HIST>
LC_DEVICE void conv_keep4(const ConvIn& a, const RowSeq& s, float* st) {
  for (int c = threadIdx.x * 4; c < a.C; c += 1024) {
    float4 in[HIST];
#pragma unroll
    for (int j = 0; j < HIST; ++j) {
      const int k = s.rows - HIST + j;
      in[j] = make_float4(0.f, 0.f, 0.f, 0.f);
      if (k >= 0) in[j] = *reinterpret_cast<const float4*>(a.x + static_cast<size_t>(s.first + k) * a.ld + c);
      else if (!s.fresh) in[j] = *reinterpret_cast<const float4*>(st + static_cast<size_t>(k + HIST) * a.C + c);
    }
#pragma unroll
    for (int j = 0; j < HIST; ++j) *reinterpret_cast<float4*>(st + static_cast<size_t>(j) * a.C + c) = in[j];
  }
}

LC_DEVICE void conv_keep(const ConvIn& a, const RowSeq& s, float* st) {
  const int hist = a.taps - 1;
  if (a.vec && hist == 1) return conv_keep4<1>(a, s, st);
  if (a.vec && hist == 2) return conv_keep4<2>(a, s, st);
  if (a.vec && hist == 3) return conv_keep4<3>(a, s, st);
  for (int c = threadIdx.x; c < a.C; c += 256)
    for (int j = 0; j < hist; ++j) {                 // (row j + rows is read before row j + 1 is written)
      const int k = s.rows - hist + j;
      float in = 0.f;
      if (k >= 0) in = a.x[static_cast<size_t>(s.first + k) * a.ld + c];
      else if (!s.fresh) in = st[static_cast<size_t>(k + hist) * a.C + c];
      st[static_cast<size_t>(j) * a.C + c] = in;
    }
}

}  // namespace
