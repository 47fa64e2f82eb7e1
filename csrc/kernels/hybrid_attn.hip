// Attention of prompt portions over a paged bf16 cache at head widths in whole groups of MFMA steps: the fast form of
// attn_tile_kernel (hybrid.hip) for masks that are an interval per row (all earlier keys, a window, a chunk). Scores, weights
// and sums are fp32 on v_mfma_f32_16x16x4_f32; only the cached keys and values are 16-bit numbers.
//
// A block is four waves = 64 query rows of ONE sequence and ONE query head, 16 rows a wave; keys come 32 at a time.
//   - A wave's queries stay in registers (scaled by scale * log2 e, so that weights are powers of two).
//   - Keys and values go to LDS as they lie in the cache (16-byte copies) and become fp32 when an operand is read: the vector
//     ALU has room between matrix instructions of 32 cycles, LDS and its bandwidth are halved, and two buffers fit, so that
//     there is one barrier per 32 keys. The loads of the next keys are in flight meanwhile.
//   - Which depth indices meet in one MFMA is free as long as both operands agree: indices 16 kk + 4 (lane >> 4) + i for
//     i = 0..3, so that an operand's four numbers come in one access. A lane's four neighbouring value columns belong to four
//     accumulator tiles for the same reason.
//   - Tiles that every row of the wave sees whole need no mask; accumulators are rescaled only when a maximum moved.
//   - GROUPS = 2: eight waves, of which the second four take every other tile of keys for the same rows; the two results are
//     joined at the end. One wave alone leaves a SIMD idle more than half of the time, and the last rows' block, which has
//     twice the mean number of keys, decides how long a small launch takes: two groups halve its chain.
#include "hybrid_common.h"

namespace {

constexpr float kLog2e = 1.4426950408889634f;

template <int N>
LC_DEVICE float rotate16(float v) {                  // inside the 16 lanes of a DPP row
  const int b = __builtin_bit_cast(int, v);
  return __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(b, b, 0x120 + N, 0xf, 0xf, false));
}
LC_DEVICE float max16(float v) {
  v = fmaxf(v, rotate16<8>(v));
  v = fmaxf(v, rotate16<4>(v));
  v = fmaxf(v, rotate16<2>(v));
  return fmaxf(v, rotate16<1>(v));
}
LC_DEVICE float sum16(float v) {
  v += rotate16<8>(v);
  v += rotate16<4>(v);
  v += rotate16<2>(v);
  return v + rotate16<1>(v);
}

LC_DEVICE float4 widen4(const uint2& w) {
  return make_float4(__uint_as_float(w.x << 16), __uint_as_float(w.x & 0xffff0000u), __uint_as_float(w.y << 16),
                     __uint_as_float(w.y & 0xffff0000u));
}

struct TileArgs {
  const float* q;                // [T, H * D]
  const bf16_t* kc;              // planes [blocks, G, BS, k_ld], [blocks, G / v_share, BS, v_ld]
  const bf16_t* vc;
  const int32_t* block_tables;
  int MB;
  const int32_t* cu_q;
  const int32_t* positions;
  void* out;                     // row (t, h) at t * o_row + h * o_ld
  int H, G, BS;
  float scale;
  int chunk, window, k_ld, v_ld, v_share;
  const float* sinks;            // score of a silent extra entry per head (null: none)
  const float* gate;             // logits [T, ld_gate], column h: the head's result times its sigmoid (null: none)
  int ld_gate;
  float out_scale;
  int o_row, o_ld;
};

constexpr int kKeys = 32;

// LDS of one group of four waves: two buffers of keys and values, the weights of four waves.
template <int DT, int VT>
constexpr int group_lds() {
  return 2 * kKeys * (16 * DT + 8 + 16 * VT + 16) * 2 + 4 * 16 * (kKeys + 4) * 4;
}

template <bool AF32, int DT, int VT, int GROUPS>
__global__ __launch_bounds__(256 * GROUPS, 2) void attn_keys32_kernel(TileArgs a) {
  constexpr int D = 16 * DT, NC = 16 * VT;
  constexpr int KS = D + 8, VS = NC + 16;            // row strides (bf16): 16 operand rows in different banks
  constexpr int PS = kKeys + 4;
  constexpr int KU = kKeys * D / 8 / 256, VU = kKeys * NC / 8 / 256;      // 16-byte units of a tile per thread
  static_assert(KU >= 1 && VU >= 1 && VT % 4 == 0, "tiles of at least one unit per thread");
  extern __shared__ __attribute__((aligned(16))) char lds[];
  const int tid = threadIdx.x & 255, group = threadIdx.x >> 8;
  bf16_t* Ks = reinterpret_cast<bf16_t*>(lds + group * group_lds<DT, VT>());      // [2][kKeys * KS]
  bf16_t* Vs = Ks + 2 * kKeys * KS;                  // [2][kKeys * VS]
  float* Ps = reinterpret_cast<float*>(Vs + 2 * kKeys * VS);                      // [4][16 * PS]
  const int b = blockIdx.z, h = GROUPS == 1 ? blockIdx.y : blockIdx.x;
  const int q0 = a.cu_q[b], q1 = a.cu_q[b + 1];
  int tile;
  if (GROUPS == 1) {
    // A portion's later rows see more keys. Workgroups i and i + 256 share a CU, so every other 256 walk the row tiles
    // backwards: a long tile and a short one meet on a CU instead of two long ones.
    const bool forward = (((b * static_cast<int>(gridDim.y) + h) * static_cast<int>(gridDim.x)) >> 8) & 1;
    tile = forward ? blockIdx.x : gridDim.x - 1 - blockIdx.x;
  } else {
    tile = gridDim.y - 1 - blockIdx.y;               // a block has a CU to itself: the long tiles of all heads first
  }
  const int row0 = q0 + tile * 64;
  if (row0 >= q1) return;                            // the same for the whole block
  const int wave = tid >> 6, lane = threadIdx.x & 63, lr = lane & 15, lk = lane >> 4;
  const int g = h / (a.H / a.G), gv = g / a.v_share, GV = a.G / a.v_share;
  const int32_t* table = a.block_tables + static_cast<size_t>(b) * a.MB;
  const int p0 = a.positions[row0];                  // rows of a portion are consecutive positions
  const int nrows = min(64, q1 - row0);
  auto first_key = [&](int p) {
    int lo = 0;
    if (a.chunk > 0) lo = (p / a.chunk) * a.chunk;
    if (a.window > 0) lo = max(lo, p - a.window + 1);
    return lo;
  };
  const int hi = p0 + nrows - 1;                     // the block's last key
  const int pw0 = p0 + 16 * wave;
  const int wave_rows = max(0, min(16, nrows - 16 * wave));
  const int wave_lo = first_key(pw0), wave_hi = pw0 + wave_rows - 1;
  const int full_lo = first_key(pw0 + 15);           // from here on to pw0 every row of the wave sees every key
  int row_lo[4];                                     // of the four rows whose scores this lane holds
#pragma unroll
  for (int r = 0; r < 4; ++r) row_lo[r] = first_key(pw0 + 4 * lk + r);
  float4 q[DT];
  {
    const bool on = lr < wave_rows;                  // (rows past the portion: zero, never stored)
    const float* src = a.q + (static_cast<size_t>(row0 + 16 * wave + (on ? lr : 0)) * a.H + h) * D + 4 * lk;
    const float s = on ? a.scale * kLog2e : 0.f;
#pragma unroll
    for (int kk = 0; kk < DT; ++kk) {
      const float4 v = *reinterpret_cast<const float4*>(src + 16 * kk);
      q[kk] = make_float4(v.x * s, v.y * s, v.z * s, v.w * s);
    }
  }
  // staging: a tile's keys lie in one block of the cache (its size is a multiple of 32)
  u32x4 kr[KU], vr[VU];
  auto block_of = [&](int j0) { return j0 <= hi ? table[j0 / a.BS] : 0; };
  auto fetch = [&](int j0, int block) {
    const bf16_t* k = a.kc + ((static_cast<size_t>(block) * a.G + g) * a.BS + j0 % a.BS) * a.k_ld;
    const bf16_t* v = a.vc + ((static_cast<size_t>(block) * GV + gv) * a.BS + j0 % a.BS) * a.v_ld;
#pragma unroll
    for (int i = 0; i < KU; ++i) {
      const int u = tid + 256 * i;                   // (keys past hi are cells of the same block: read, never seen)
      kr[i] = *reinterpret_cast<const u32x4*>(k + (u / (D / 8)) * a.k_ld + (u % (D / 8)) * 8);
    }
#pragma unroll
    for (int i = 0; i < VU; ++i) {
      const int u = tid + 256 * i;
      vr[i] = *reinterpret_cast<const u32x4*>(v + (u / (NC / 8)) * a.v_ld + (u % (NC / 8)) * 8);
    }
  };
  auto stage = [&](int buf, int j0) {                // (the first use of what fetch loaded)
    if (j0 + kKeys - 1 > hi) {
#pragma unroll
      for (int i = 0; i < VU; ++i)                   // what nobody wrote may be no number, and its weight of zero times it
        if (j0 + (tid + 256 * i) / (NC / 8) > hi) vr[i] = u32x4{0u, 0u, 0u, 0u};
    }
#pragma unroll
    for (int i = 0; i < KU; ++i) {
      const int u = tid + 256 * i;
      *reinterpret_cast<u32x4*>(&Ks[buf * kKeys * KS + (u / (D / 8)) * KS + (u % (D / 8)) * 8]) = kr[i];
    }
#pragma unroll
    for (int i = 0; i < VU; ++i) {
      const int u = tid + 256 * i;
      *reinterpret_cast<u32x4*>(&Vs[buf * kKeys * VS + (u / (NC / 8)) * VS + (u % (NC / 8)) * 8]) = vr[i];
    }
  };
  float m[4], l[4];
  f32x4 o[VT];
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    m[r] = a.sinks != nullptr && group == 0 ? a.sinks[h] * kLog2e : -INFINITY;
    l[r] = a.sinks != nullptr && group == 0 && lr == 0 ? 1.f : 0.f;
  }
#pragma unroll
  for (int t = 0; t < VT; ++t) o[t] = f32x4{0.f, 0.f, 0.f, 0.f};
  float* Pw = Ps + wave * 16 * PS;
  constexpr int STEP = kKeys * GROUPS;
  const int lo_tile = (first_key(p0) / kKeys) * kKeys;
  int j0 = lo_tile + group * kKeys;                  // this group's first tile
  if (j0 <= hi) {
    fetch(j0, block_of(j0));
    stage(0, j0);
  }
  int ahead = block_of(j0 + STEP), buf = 0;
  for (int jb = lo_tile; jb <= hi; jb += STEP, j0 += STEP, buf ^= 1) {      // (all groups take the same number of turns)
    __syncthreads();                                 // this tile is in place, and nobody reads the other buffer any more
    const bool more = j0 + STEP <= hi;
    if (more) {
      fetch(j0 + STEP, ahead);
      ahead = block_of(j0 + 2 * STEP);
    }
    if (wave_rows > 0 && j0 <= wave_hi && j0 + kKeys - 1 >= wave_lo) {      // wave-uniform
      f32x4 s[2][2];
#pragma unroll
      for (int e = 0; e < 2; ++e) s[e][0] = s[e][1] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int kk = 0; kk < DT; ++kk)
#pragma unroll
        for (int e = 0; e < 2; ++e) {
          const float4 k = widen4(*reinterpret_cast<const uint2*>(&Ks[buf * kKeys * KS + (16 * e + lr) * KS + 16 * kk + 4 * lk]));
          s[e][0] = __builtin_amdgcn_mfma_f32_16x16x4f32(q[kk].x, k.x, s[e][0], 0, 0, 0);
          s[e][1] = __builtin_amdgcn_mfma_f32_16x16x4f32(q[kk].y, k.y, s[e][1], 0, 0, 0);
          s[e][0] = __builtin_amdgcn_mfma_f32_16x16x4f32(q[kk].z, k.z, s[e][0], 0, 0, 0);
          s[e][1] = __builtin_amdgcn_mfma_f32_16x16x4f32(q[kk].w, k.w, s[e][1], 0, 0, 0);
        }
      float sv[2][4];
#pragma unroll
      for (int e = 0; e < 2; ++e)
#pragma unroll
        for (int r = 0; r < 4; ++r) sv[e][r] = s[e][0][r] + s[e][1][r];
      if (j0 + kKeys - 1 > pw0 || j0 < full_lo) {    // some row does not see the whole tile
#pragma unroll
        for (int e = 0; e < 2; ++e)
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            const int j = j0 + 16 * e + lr;
            if (j > pw0 + 4 * lk + r || j < row_lo[r]) sv[e][r] = -INFINITY;
          }
      }
      float corr[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float mn = fmaxf(m[r], max16(fmaxf(sv[0][r], sv[1][r])));
        const float base = mn == -INFINITY ? 0.f : mn;        // nothing visible yet: weights 0, no NaN
        corr[r] = fast_exp2(m[r] - base);
        const float pa = fast_exp2(sv[0][r] - base), pb = fast_exp2(sv[1][r] - base);
        l[r] = l[r] * corr[r] + pa + pb;             // this lane's keys only: summed over the row at the end
        m[r] = mn;
        Pw[(4 * lk + r) * PS + lr] = pa;
        Pw[(4 * lk + r) * PS + 16 + lr] = pb;
      }
      if (__any(corr[0] != 1.f || corr[1] != 1.f || corr[2] != 1.f || corr[3] != 1.f)) {
#pragma unroll
        for (int t = 0; t < VT; ++t)
#pragma unroll
          for (int r = 0; r < 4; ++r) o[t][r] *= corr[r];
      }
      // P goes from the score layout to the operand layout through this wave's own LDS patch: the wave's LDS accesses
      // execute in order, the fences keep the compiler from moving them
      __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
      __builtin_amdgcn_wave_barrier();
      __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
#pragma unroll
      for (int e = 0; e < 2; ++e) {
        const float4 p = *reinterpret_cast<const float4*>(Pw + lr * PS + 16 * e + 4 * lk);
#pragma unroll
        for (int t = 0; t < VT; t += 4) {
          float4 v[4];
#pragma unroll
          for (int i = 0; i < 4; ++i)
            v[i] = widen4(*reinterpret_cast<const uint2*>(&Vs[buf * kKeys * VS + (16 * e + 4 * lk + i) * VS + t * 16 + 4 * lr]));
          const float pi[4] = {p.x, p.y, p.z, p.w};
#pragma unroll
          for (int i = 0; i < 4; ++i) {              // four independent chains
            o[t] = __builtin_amdgcn_mfma_f32_16x16x4f32(pi[i], v[i].x, o[t], 0, 0, 0);
            o[t + 1] = __builtin_amdgcn_mfma_f32_16x16x4f32(pi[i], v[i].y, o[t + 1], 0, 0, 0);
            o[t + 2] = __builtin_amdgcn_mfma_f32_16x16x4f32(pi[i], v[i].z, o[t + 2], 0, 0, 0);
            o[t + 3] = __builtin_amdgcn_mfma_f32_16x16x4f32(pi[i], v[i].w, o[t + 3], 0, 0, 0);
          }
        }
      }
      __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");     // P is read before the next tile overwrites it
      __builtin_amdgcn_wave_barrier();
    }
    if (more) stage(buf ^ 1, j0 + STEP);
  }
  if constexpr (GROUPS == 2) {
    // the second group's sums go through LDS (the tiles are done with), register after register, to the first one's lanes
    static_assert((4 * VT + 8) * 256 * 4 <= 2 * group_lds<DT, VT>(), "the sums fit where the tiles were");
    float* xs = reinterpret_cast<float*>(lds);
    __syncthreads();
    if (group == 1) {
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        xs[r * 256 + tid] = m[r];
        xs[(4 + r) * 256 + tid] = l[r];
      }
#pragma unroll
      for (int t = 0; t < VT; ++t)
#pragma unroll
        for (int r = 0; r < 4; ++r) xs[(8 + 4 * t + r) * 256 + tid] = o[t][r];
    }
    __syncthreads();
    if (group == 1) return;                          // (no barrier follows)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const float m1 = xs[r * 256 + tid], mn = fmaxf(m[r], m1);
      const float base = mn == -INFINITY ? 0.f : mn;
      const float f0 = fast_exp2(m[r] - base), f1 = fast_exp2(m1 - base);
      l[r] = l[r] * f0 + xs[(4 + r) * 256 + tid] * f1;
#pragma unroll
      for (int t = 0; t < VT; ++t) o[t][r] = o[t][r] * f0 + xs[(8 + 4 * t + r) * 256 + tid] * f1;
    }
  }
  typedef typename Act<AF32>::type act_t;
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int row = 4 * lk + r;
    const float sum = sum16(l[r]);
    if (row >= wave_rows) continue;
    const size_t tok = static_cast<size_t>(row0) + 16 * wave + row;
    const float fin = a.out_scale * (a.gate != nullptr ? sigmoidf_(a.gate[tok * a.ld_gate + h]) : 1.f) / sum;
    act_t* dst = static_cast<act_t*>(a.out) + tok * a.o_row + static_cast<size_t>(h) * a.o_ld + 4 * lr;
#pragma unroll
    for (int t = 0; t < VT; t += 4)
      store_act4<AF32>(dst, 16 * t, make_float4(o[t][r] * fin, o[t + 1][r] * fin, o[t + 2][r] * fin, o[t + 3][r] * fin));
  }
}

}  // namespace

// Launches of up to this many row tiles run two groups of waves per tile.
constexpr long long kTwoGroupBlocks = 1024;

// Whether lc_attn_keys32 takes the shape (1) or not (0).
LC_EXPORT int lc_attn_keys32_ok(int D, int Dv, int BS) {
  return BS % kKeys == 0 && ((D == 64 && (Dv == 64 || Dv == 128)) || (D == 128 && (Dv == 128 || Dv == 256)));
}

// Sequences [0, n_seq) of cu_q, the longest of max_len rows; planes, row strides and options as for lc_attn_tile.
LC_EXPORT int lc_attn_keys32(const void* q, const void* kc, const void* vc, const void* block_tables, int MB, const void* cu_q,
                             const void* positions, void* out, int act_f32, int n_seq, int max_len, int H, int G, int D, int Dv,
                             int BS, float scale, int chunk, int window, int k_ld, int v_ld, const void* sinks, const void* gate,
                             int ld_gate, float out_scale, int o_row, int v_share, int o_ld, hipStream_t st) {
  if (n_seq <= 0 || max_len <= 0) return 0;
  if (H <= 0 || G <= 0 || H % G || MB <= 0 || v_share <= 0 || G % v_share || !lc_attn_keys32_ok(D, Dv, BS)) return -1;
  if (k_ld < D || v_ld < Dv || k_ld % 8 || v_ld % 8 || !aligned16(q) || !aligned16(kc) || !aligned16(vc)) return -1;
  if (o_ld < Dv || o_row < H * o_ld || o_ld % 4 || o_row % 4 || reinterpret_cast<uintptr_t>(out) % (act_f32 ? 16 : 8)) return -1;
  if (gate != nullptr && ld_gate < H) return -1;
  const TileArgs a{static_cast<const float*>(q), static_cast<const bf16_t*>(kc), static_cast<const bf16_t*>(vc),
                   static_cast<const int32_t*>(block_tables), MB, static_cast<const int32_t*>(cu_q),
                   static_cast<const int32_t*>(positions), out, H, G, BS, scale, chunk, window, k_ld, v_ld, v_share,
                   static_cast<const float*>(sinks), static_cast<const float*>(gate), ld_gate, out_scale, o_row, o_ld};
  const int tiles = (max_len + 63) / 64;
  const bool two = static_cast<long long>(tiles) * H * n_seq <= kTwoGroupBlocks;
#define LC_K32_G(A32, DT, VT)                                                                                             \
  do {                                                                                                                    \
    constexpr int one_lds = group_lds<DT, VT>();                                                                          \
    static LcDeviceOnce attr_once;                                                                                        \
    attr_once.run([&] {                                                                                                   \
      (void)hipFuncSetAttribute(reinterpret_cast<const void*>(attn_keys32_kernel<A32, DT, VT, 1>),                        \
                                hipFuncAttributeMaxDynamicSharedMemorySize, one_lds);                                     \
      (void)hipFuncSetAttribute(reinterpret_cast<const void*>(attn_keys32_kernel<A32, DT, VT, 2>),                        \
                                hipFuncAttributeMaxDynamicSharedMemorySize, 2 * one_lds);                                 \
    });                                                                                                                   \
    if (two) attn_keys32_kernel<A32, DT, VT, 2><<<dim3(H, tiles, n_seq), dim3(512), 2 * one_lds, st>>>(a);                \
    else attn_keys32_kernel<A32, DT, VT, 1><<<dim3(tiles, H, n_seq), dim3(256), one_lds, st>>>(a);                        \
  } while (0)
#define LC_K32(DT, VT)                        \
  do {                                        \
    if (act_f32) LC_K32_G(true, DT, VT);      \
    else LC_K32_G(false, DT, VT);             \
  } while (0)
  if (D == 64 && Dv == 64) LC_K32(4, 4);
  else if (D == 64) LC_K32(4, 8);
  else if (Dv == 128) LC_K32(8, 8);
  else LC_K32(8, 16);
#undef LC_K32
#undef LC_K32_G
  LC_RETURN_LAST_ERROR();
}
