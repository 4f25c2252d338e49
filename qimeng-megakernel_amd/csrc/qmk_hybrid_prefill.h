// Prefill kernels of the hybrid route: a portion of M tokens, one launch per fused operation.
//
// Element type T (bf16 or fp32) is that of the activations between kernels; sums, norms, angles, scores, gates,
// recurrences and the residual streams are fp32 in both.  Weights are bf16 in memory in both: in fp32 mode they are
// widened in registers and multiplied by the fp32 matrix instructions.
#pragma once

#include "qmk_hybrid_ops.h"

namespace qmk {
namespace hybrid {

constexpr int kPfThreads = 256;

enum : int {
  EPI_STORE = 0,        // out T [m][ldo]
  EPI_RGLRU_IN,         // gelu of the y half, bias on both
  EPI_LRU_GATES,        // (r, i) pairs -> decay a and input b of the recurrence
  EPI_LATENT_IN,        // rotation of q, sigmoid of the gate, raw latent
  EPI_RESIDUAL,         // all streams of the residual and the next sublayer's input
  EPI_GEGLU,            // (gate, up) pairs
  EPI_WKV_IN,           // r, k, v fp32; silu gate; tanh
  EPI_WKV_DECAY,        // exp(-exp(. + w0))
  EPI_LOGITS,
  EPI_CAPPED_LOGITS,    // logits times a constant, softly capped
  EPI_ADD,              // onto the fp32 residual
  EPI_ATTENTION_IN,     // rotation of q and k, k and v into the cache, sigmoid of the gate
  EPI_DELTA_IN,         // q, k, v fp32; raw ranks; sigmoid of the step sizes
  EPI_DELTA_DECAY,
  EPI_SIGMOID,
  EPI_GLA_IN,           // q, k, v fp32; silu gate; raw rank
  EPI_GLA_DECAY,
};

struct GemmArgs {
  const void* a;         // TA [M][lda]
  const void* w;         // TW [N][ldw]
  int M, N, K, lda, ldw, groups, last_n;   // group g: a + g a_step, w + g w_step, N rows (the last: last_n)
  long long a_step, w_step;
  int epi;
  void* out;             // meaning by epilogue
  void* out2;
  float* f0;
  float* f1;
  const void* src;
  int ldo;
  QmkHybridLayer layer;
  int down, first, position, streams, width, rows_cap, slot;
  float logit_scale, logit_softcap;
  const float* next;
};

template <class T>
__device__ __forceinline__ void store4(T* at, f32x4 v) {
  if constexpr (sizeof(T) == 2) {
    *reinterpret_cast<uint2*>(at) = make_uint2(f2bf2(v[0], v[1]), f2bf2(v[2], v[3]));
  } else {
    *reinterpret_cast<f32x4*>(at) = v;
  }
}
template <class T>
__device__ __forceinline__ f32x4 read4(const T* at) {
  if constexpr (sizeof(T) == 2) {
    const uint2 t = *reinterpret_cast<const uint2*>(at);
    return f32x4{bf_lo(t.x), bf_hi(t.x), bf_lo(t.y), bf_hi(t.y)};
  } else {
    return *reinterpret_cast<const f32x4*>(at);
  }
}

// Four consecutive outputs n .. n+3 of token m.
template <class T>
__device__ __forceinline__ void epilogue(const GemmArgs& g, int group, int m, int n, f32x4 v) {
  const QmkHybridLayer& l = g.layer;
  switch (g.epi) {
    case EPI_STORE: store4(static_cast<T*>(g.out) + static_cast<size_t>(m) * g.ldo + n, v); break;
    case EPI_RGLRU_IN: {
      const f32x4 b = *reinterpret_cast<const f32x4*>(l.in_b + n);
      v += b;
      if (n < l.mix_width) {
#pragma unroll
        for (int i = 0; i < 4; ++i) v[i] = gelu_tanh(v[i]);
        store4(static_cast<T*>(g.out) + static_cast<size_t>(m) * l.mix_width + n, v);
      } else {
        store4(static_cast<T*>(g.out2) + static_cast<size_t>(m) * l.mix_width + n - l.mix_width, v);
      }
      break;
    }
    case EPI_LRU_GATES: {
      const f32x4 b = *reinterpret_cast<const f32x4*>(l.mid_b + static_cast<size_t>(group) * 2 * l.block_dim + n);
      v += b;
      const int c = group * l.block_dim + n / 2;
      const size_t at = static_cast<size_t>(m) * l.mix_width + c;
      const T* u = static_cast<const T*>(g.src) + at;
      float2 a2, b2;
      {
        const float la = sigmoid(v[0]) * l.vec0[c];
        a2.x = expf(la);
        b2.x = sqrtf(-expm1f(2.f * la)) * sigmoid(v[1]) * to_f32(u[0]);
      }
      {
        const float la = sigmoid(v[2]) * l.vec0[c + 1];
        a2.y = expf(la);
        b2.y = sqrtf(-expm1f(2.f * la)) * sigmoid(v[3]) * to_f32(u[1]);
      }
      *reinterpret_cast<float2*>(g.f0 + at) = a2;
      *reinterpret_cast<float2*>(g.f1 + at) = b2;
      break;
    }
    case EPI_LATENT_IN: {
      const int q_rows = l.heads * l.q_stride, g_rows = l.heads * l.v_dim;
      if (n < q_rows) {
        const int d = n % l.q_stride - l.head_dim;
        if (d >= 0) {
          float e[4] = {v[0], v[1], v[2], v[3]};
          rotate(l, g.position + m, d, e[0], e[1]);
          rotate(l, g.position + m, d + 2, e[2], e[3]);
          v = f32x4{e[0], e[1], e[2], e[3]};
        }
        store4(static_cast<T*>(g.out) + static_cast<size_t>(m) * q_rows + n, v);
      } else if (n < q_rows + g_rows) {
#pragma unroll
        for (int i = 0; i < 4; ++i) v[i] = sigmoid(v[i]);
        store4(static_cast<T*>(g.out2) + static_cast<size_t>(m) * g_rows + n - q_rows, v);
      } else {
        store4(g.f0 + static_cast<size_t>(m) * (l.rank + l.rot_dim) + n - q_rows - g_rows, v);
      }
      break;
    }
    case EPI_RESIDUAL: {
      const int S = g.streams, D = g.width;
      const float* hc = l.hc + (g.down ? S * (S + 2) : 0);
      float* x = g.f0 + static_cast<size_t>(m) * S * D + n;
      f32x4 old[kMaxStreams];
#pragma unroll
      for (int s = 0; s < kMaxStreams; ++s)
        if (s < S) old[s] = *reinterpret_cast<const f32x4*>(x + static_cast<size_t>(s) * D);
      f32x4 u = {};
#pragma unroll
      for (int t = 0; t < kMaxStreams; ++t) {
        if (t < S) {
          f32x4 now = v * hc[S + t];
#pragma unroll
          for (int s = 0; s < kMaxStreams; ++s)
            if (s < S) now += old[s] * hc[2 * S + s * S + t];
          *reinterpret_cast<f32x4*>(x + static_cast<size_t>(t) * D) = now;
          u += now * g.next[t];
        }
      }
      *reinterpret_cast<f32x4*>(g.f1 + static_cast<size_t>(m) * D + n) = u;
      break;
    }
    case EPI_GEGLU: {
      T* o = static_cast<T*>(g.out) + static_cast<size_t>(m) * l.ff + n / 2;
      const bool silu = l.act == QMK_ACT_SILU;
      const float a = (silu ? v[0] * sigmoid(v[0]) : gelu_tanh(v[0])) * v[1], b = (silu ? v[2] * sigmoid(v[2]) : gelu_tanh(v[2])) * v[3];
      if constexpr (sizeof(T) == 2) *reinterpret_cast<uint32_t*>(o) = f2bf2(a, b);
      else *reinterpret_cast<float2*>(o) = make_float2(a, b);
      break;
    }
    case EPI_WKV_IN: {
      const int N = l.heads * l.head_dim;
      if (group < 3) {
        store4(g.f0 + (static_cast<size_t>(group) * g.rows_cap + m) * N + n, v);
      } else if (group == 3) {
#pragma unroll
        for (int i = 0; i < 4; ++i) v[i] *= sigmoid(v[i]);
        store4(static_cast<T*>(g.out) + static_cast<size_t>(m) * N + n, v);
      } else {
#pragma unroll
        for (int i = 0; i < 4; ++i) v[i] = tanhf(v[i]);
        store4(static_cast<T*>(g.out2) + static_cast<size_t>(m) * l.rank + n, v);
      }
      break;
    }
    case EPI_WKV_DECAY: {
      const f32x4 b = *reinterpret_cast<const f32x4*>(l.mid_b + n);
#pragma unroll
      for (int i = 0; i < 4; ++i) v[i] = expf(-expf(v[i] + b[i]));
      store4(g.f0 + static_cast<size_t>(m) * g.ldo + n, v);
      break;
    }
    case EPI_CAPPED_LOGITS: {
#pragma unroll
      for (int i = 0; i < 4; ++i) v[i] = soft_cap(v[i] * g.logit_scale, g.logit_softcap);
      store4(g.f0 + static_cast<size_t>(m) * g.ldo + n, v);
      break;
    }
    case EPI_ADD: {
      float* x = g.f0 + static_cast<size_t>(m) * g.ldo + n;
      store4(x, read4(x) + v);
      break;
    }
    case EPI_ATTENTION_IN: {
      const int q_rows = l.heads * l.q_stride, k_rows = l.kv_heads * l.head_dim, v_rows = l.kv_heads * l.v_dim, row = l.head_dim + l.v_dim, pos = g.position + m;
      T* cache = static_cast<T*>(l.cache) + (static_cast<size_t>(g.slot) * l.ring + pos % l.ring) * l.kv_heads * row;
      if (n < q_rows + k_rows) {
        const int d = n < q_rows ? n % l.q_stride : (n - q_rows) % l.head_dim;
        float e[4] = {v[0], v[1], v[2], v[3]};
        rotate(l, pos, d, e[0], e[1]);
        rotate(l, pos, d + 2, e[2], e[3]);
        v = f32x4{e[0], e[1], e[2], e[3]};
        store4(n < q_rows ? static_cast<T*>(g.out) + static_cast<size_t>(m) * q_rows + n : cache + (n - q_rows) / l.head_dim * row + d, v);
      } else if (n < q_rows + k_rows + v_rows) {
        const int c = n - q_rows - k_rows;
        store4(cache + c / l.v_dim * row + l.head_dim + c % l.v_dim, v);
      } else {
#pragma unroll
        for (int i = 0; i < 4; ++i) v[i] = sigmoid(v[i]);
        store4(static_cast<T*>(g.out2) + static_cast<size_t>(m) * l.mix_width + n - q_rows - k_rows - v_rows, v);
      }
      break;
    }
    case EPI_DELTA_IN: {
      const int channels = conv_channels(l), ranks = l.rank + l.gate_rank;
      if (n < channels) {
        store4(g.f1 + static_cast<size_t>(m) * channels + n, v);
      } else if (n < channels + ranks) {
        store4(static_cast<T*>(g.out2) + static_cast<size_t>(m) * ranks + n - channels, v);
      } else {
#pragma unroll
        for (int i = 0; i < 4; ++i) v[i] = sigmoid(v[i]);
        store4(g.f0 + static_cast<size_t>(m) * g.ldo + n - channels - ranks, v);
      }
      break;
    }
    case EPI_DELTA_DECAY: {
      const f32x4 b = *reinterpret_cast<const f32x4*>(l.mid_b + n);
#pragma unroll
      for (int i = 0; i < 4; ++i) v[i] = delta_decay(l, n / l.head_dim, v[i] + b[i]);
      store4(g.f0 + static_cast<size_t>(m) * g.ldo + n, v);
      break;
    }
    case EPI_SIGMOID: {
#pragma unroll
      for (int i = 0; i < 4; ++i) v[i] = sigmoid(v[i]);
      store4(static_cast<T*>(g.out) + static_cast<size_t>(m) * g.ldo + n, v);
      break;
    }
    case EPI_GLA_IN: {
      const int qkv = 2 * l.heads * l.head_dim + l.mix_width;
      if (n < qkv) {
        store4(g.f0 + static_cast<size_t>(m) * qkv + n, v);
      } else if (n < qkv + l.mix_width) {
#pragma unroll
        for (int i = 0; i < 4; ++i) v[i] *= sigmoid(v[i]);
        store4(static_cast<T*>(g.out) + static_cast<size_t>(m) * l.mix_width + n - qkv, v);
      } else {
        store4(static_cast<T*>(g.out2) + static_cast<size_t>(m) * l.rank + n - qkv - l.mix_width, v);
      }
      break;
    }
    case EPI_GLA_DECAY: {
      const f32x4 b = *reinterpret_cast<const f32x4*>(l.mid_b + n);
#pragma unroll
      for (int i = 0; i < 4; ++i) v[i] = gla_decay(l, v[i] + b[i]);
      store4(g.f0 + static_cast<size_t>(m) * g.ldo + n, v);
      break;
    }
    default: store4(g.f0 + static_cast<size_t>(m) * g.ldo + n, v); break;
  }
}

// A workgroup's accumulators -> epilogue, through LDS (a wave's own part, quads of a row exchanged by its number): a lane's
// accumulators are then read back in a loop, and the lanes of a row write neighbouring outputs of one token.
template <class T, int BM, int BN, int kTn, int kTm>
__device__ __forceinline__ void finish_tile(const GemmArgs& g, int group, int m0, int n0, int N, v4u* lds, const f32x4 (&acc)[kTn][kTm]) {
  constexpr int kWm = BM / 2, kWn = BN / 2, kQuads = kWn / 4;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, wm = wave & 1, wn = wave >> 1;
  f32x4* out = reinterpret_cast<f32x4*>(lds) + wave * kWm * kQuads;
#pragma unroll
  for (int i = 0; i < kTm; ++i)
#pragma unroll
    for (int j = 0; j < kTn; ++j) {
      const int m = i * 16 + (lane & 15), quad = j * 4 + (lane >> 4);
      out[m * kQuads + (quad ^ (m & (kQuads - 1)))] = acc[j][i];
    }
#pragma unroll 1
  for (int id = lane; id < kWm * kQuads; id += 64) {
    const int r = id / kQuads, quad = id % kQuads, m = m0 + wm * kWm + r, n = n0 + wn * kWn + quad * 4;
    if (m < g.M && n < N) epilogue<T>(g, group, m, n, out[r * kQuads + (quad ^ (r & (kQuads - 1)))]);
  }
}

// Until at most `n` of this wave's vector-memory requests are outstanding and none of its LDS reads.
template <int n>
__device__ __forceinline__ void wait_outstanding() {
  static_assert(n >= 0 && n < 64, "six bits");
  asm volatile("s_waitcnt vmcnt(%0) lgkmcnt(0)" ::"n"(n) : "memory");
}

// out[m][n] = sum_k a[m][k] w[n][k]: BN weight rows x BM tokens per workgroup, four waves as 2 x 2, 64 columns a step.
// The weights are the matrix instruction's first operand, so a lane ends up with four consecutive outputs of one token.
// LDS tiles hold 16-byte units, a row's units rotated by the row number (conflict-free fragment reads).
template <class TA, class TW, class T, int BM, int BN>
__global__ __launch_bounds__(kPfThreads) void gemm(const GemmArgs g) {
  constexpr int kBK = 64;
  constexpr int kUnitA = 16 / sizeof(TA), kUnitW = 16 / sizeof(TW);       // elements of a unit
  constexpr int kRowA = kBK / kUnitA, kRowW = kBK / kUnitW;                // units of a row
  constexpr int kLoadsA = BM * kRowA / kPfThreads, kLoadsW = BN * kRowW / kPfThreads;
  constexpr int kTm = BM / 2 / 16, kTn = BN / 2 / 16;
  constexpr int kTileUnits = 2 * (BM * kRowA + BN * kRowW), kOutUnits = BM * BN / 4;
  __shared__ v4u lds[kTileUnits > kOutUnits ? kTileUnits : kOutUnits];
  v4u(*la)[BM * kRowA] = reinterpret_cast<v4u(*)[BM * kRowA]>(lds);
  v4u(*lw)[BN * kRowW] = reinterpret_cast<v4u(*)[BN * kRowW]>(lds + 2 * BM * kRowA);
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, wm = wave & 1, wn = wave >> 1;
  const int group = blockIdx.z;
  const int N = group == g.groups - 1 ? g.last_n : g.N;
  const int m0 = blockIdx.y * BM, n0 = blockIdx.x * BN;
  if (n0 >= N) return;
  const TA* a = static_cast<const TA*>(g.a) + group * g.a_step;
  const TW* w = static_cast<const TW*>(g.w) + group * g.w_step;

  v4u ra[kLoadsA], rw[kLoadsW];
  auto fetch = [&](int k0) {
#pragma unroll
    for (int i = 0; i < kLoadsA; ++i) {
      const int id = i * kPfThreads + tid, r = id / kRowA, c = id % kRowA, k = k0 + c * kUnitA;
      v4u z = {0u, 0u, 0u, 0u};
      ra[i] = k < g.K ? *reinterpret_cast<const v4u*>(a + static_cast<size_t>(min(m0 + r, g.M - 1)) * g.lda + k) : z;
    }
#pragma unroll
    for (int i = 0; i < kLoadsW; ++i) {
      const int id = i * kPfThreads + tid, r = id / kRowW, c = id % kRowW, k = k0 + c * kUnitW;
      v4u z = {0u, 0u, 0u, 0u};
      rw[i] = k < g.K ? *reinterpret_cast<const v4u*>(w + static_cast<size_t>(min(n0 + r, N - 1)) * g.ldw + k) : z;
    }
  };
  auto place = [](int r, int unit, int row_units) { return r * row_units + (unit ^ ((r & 7) * (row_units / 8))); };
  auto stash = [&](int buf) {
#pragma unroll
    for (int i = 0; i < kLoadsA; ++i) {
      const int id = i * kPfThreads + tid;
      la[buf][place(id / kRowA, id % kRowA, kRowA)] = ra[i];
    }
#pragma unroll
    for (int i = 0; i < kLoadsW; ++i) {
      const int id = i * kPfThreads + tid;
      lw[buf][place(id / kRowW, id % kRowW, kRowW)] = rw[i];
    }
  };
  f32x4 acc[kTn][kTm] = {};
  const int steps = (g.K + kBK - 1) / kBK;
  fetch(0);
  stash(0);
  __syncthreads();
  for (int s = 0; s < steps; ++s) {
    const int buf = s & 1;
    if (s + 1 < steps) fetch((s + 1) * kBK);
#pragma unroll
    for (int kk = 0; kk < 2; ++kk) {
      Frag<TA> fa[kTm];
      const int q = kk * 4 + (lane >> 4);      // which run of eight columns
#pragma unroll
      for (int i = 0; i < kTm; ++i) {
        const int r = wm * (BM / 2) + i * 16 + (lane & 15);
        fa[i] = load_frag(reinterpret_cast<const TA*>(&la[buf][place(r, q * (kRowA / 8), kRowA)]));
      }
#pragma unroll
      for (int j = 0; j < kTn; ++j) {
        const int r = wn * (BN / 2) + j * 16 + (lane & 15);
        const Frag<TW> fw = load_frag(reinterpret_cast<const TW*>(&lw[buf][place(r, q * (kRowW / 8), kRowW)]));
#pragma unroll
        for (int i = 0; i < kTm; ++i) acc[j][i] = mma(fw, fa[i], acc[j][i]);
      }
    }
    if (s + 1 < steps) stash(buf ^ 1);
    __syncthreads();
  }
  finish_tile<T, BM, BN>(g, group, m0, n0, N, lds, acc);
}

// The same for bf16 x bf16 with K a multiple of 64: tiles go from memory to LDS without passing through registers, STAGES
// buffers deep, so that STAGES - 1 steps are in flight while one is multiplied.
template <class T, int BM, int BN, int STAGES>
__global__ __launch_bounds__(kPfThreads) void gemm_direct(const GemmArgs g) {
  constexpr int kBK = 64, kRow = kBK / 8;                                   // a row: eight units of 16 bytes
  constexpr int kLoads = (BM + BN) * kRow / kPfThreads, kStageUnits = (BM + BN) * kRow;
  constexpr int kTm = BM / 2 / 16, kTn = BN / 2 / 16, kOutUnits = BM * BN / 4, kAhead = STAGES - 1;
  __shared__ __align__(16) v4u lds[STAGES * kStageUnits > kOutUnits ? STAGES * kStageUnits : kOutUnits];
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), wm = wave & 1, wn = wave >> 1;
  const int group = blockIdx.z;
  const int N = group == g.groups - 1 ? g.last_n : g.N;
  const int m0 = blockIdx.y * BM, n0 = blockIdx.x * BN;
  if (n0 >= N) return;
  const u16* a = static_cast<const u16*>(g.a) + group * g.a_step;
  const u16* w = static_cast<const u16*>(g.w) + group * g.w_step;

  // This thread's places in a stage: unit i * 256 + tid, tokens first.  A row's units are exchanged by its number, here on
  // the memory side: the LDS side of such a load is one run of 64 units per wave.
  const u16* from[kLoads];
#pragma unroll
  for (int i = 0; i < kLoads; ++i) {
    const int id = i * kPfThreads + tid, r = id / kRow, c = ((id % kRow) ^ (r & 7)) * 8;
    from[i] = r < BM ? a + static_cast<size_t>(min(m0 + r, g.M - 1)) * g.lda + c : w + static_cast<size_t>(min(n0 + r - BM, N - 1)) * g.ldw + c;
  }
  auto issue = [&](int buf) {
#pragma unroll
    for (int i = 0; i < kLoads; ++i) {
      const auto* src = (const __attribute__((address_space(1))) uint32_t*)from[i];
      auto* dst = (__attribute__((address_space(3))) uint32_t*)(lds + buf * kStageUnits + i * kPfThreads + wave * 64);
      __builtin_amdgcn_global_load_lds(src, dst, 16, 0, 0);
      from[i] += kBK;
    }
  };
  f32x4 acc[kTn][kTm] = {};
  const int steps = g.K / kBK;
#pragma unroll
  for (int s = 0; s < kAhead; ++s)
    if (s < steps) issue(s);
  int buf = 0;
  for (int s = 0; s < steps; ++s) {
    // Everything up to this step's stage has landed; the barrier makes that true of every wave's part, and says that the
    // buffer filled next is no longer read.
    if (s + kAhead - 1 < steps) wait_outstanding<(kAhead - 1) * kLoads>();
    else wait_outstanding<0>();
    __builtin_amdgcn_s_barrier();
    asm volatile("" ::: "memory");
    if (s + kAhead < steps) issue(buf == 0 ? STAGES - 1 : buf - 1);
    const v4u* la = lds + buf * kStageUnits;
    const v4u* lw = la + BM * kRow;
#pragma unroll
    for (int kk = 0; kk < 2; ++kk) {
      const int q = kk * 4 + (lane >> 4);
      Frag<u16> fa[kTm];
#pragma unroll
      for (int i = 0; i < kTm; ++i) {
        const int r = wm * (BM / 2) + i * 16 + (lane & 15);
        fa[i] = load_frag(reinterpret_cast<const u16*>(la + r * kRow + (q ^ (r & 7))));
      }
#pragma unroll
      for (int j = 0; j < kTn; ++j) {
        const int r = wn * (BN / 2) + j * 16 + (lane & 15);
        const Frag<u16> fw = load_frag(reinterpret_cast<const u16*>(lw + r * kRow + (q ^ (r & 7))));
#pragma unroll
        for (int i = 0; i < kTm; ++i) acc[j][i] = mma(fw, fa[i], acc[j][i]);
      }
    }
    buf = buf + 1 == STAGES ? 0 : buf + 1;
  }
  __syncthreads();
  finish_tile<T, BM, BN>(g, group, m0, n0, N, lds, acc);
}

__device__ __forceinline__ float pf_block_sum(float v, float* scratch) {
  v = wave_sum(v);
  __syncthreads();
  if ((threadIdx.x & 63) == 0) scratch[threadIdx.x >> 6] = v;
  __syncthreads();
  return scratch[0] + scratch[1] + scratch[2] + scratch[3];
}

// x = the token's embedding in every stream, u = what the first sublayer reads.
__global__ __launch_bounds__(kPfThreads) void embed_tokens(const u16* table, const int64_t* tokens, int vocab, const float* hc_in, int S, int D,
                                                           float* x, float* u) {
  const int m = blockIdx.x;
  long long t = tokens[m];
  if (t < 0 || t >= vocab) t = 0;
  const float g = weight_sum(hc_in, S);
  for (int i = threadIdx.x; i < D; i += kPfThreads) {
    const float e = bf2f(table[t * D + i]);
    for (int s = 0; s < S; ++s) x[(static_cast<size_t>(m) * S + s) * D + i] = e;
    u[static_cast<size_t>(m) * D + i] = e * g;
  }
}

// h = norm(u[row]); row = want[blockIdx.x] where given
template <class T>
__global__ __launch_bounds__(kPfThreads) void norm_rows(const float* u, const float* weight, const int32_t* want, int limit, int D, int true_width, float eps, T* h) {
  __shared__ float scratch[4];
  const int m = blockIdx.x;
  int from = want != nullptr ? want[m] : m;
  from = from < 0 || from >= limit ? 0 : from;
  const float* row = u + static_cast<size_t>(from) * D;
  float sq = 0.f;
  for (int i = threadIdx.x * 4; i < D; i += kPfThreads * 4) {
    const f32x4 v = *reinterpret_cast<const f32x4*>(row + i);
    sq += v[0] * v[0] + v[1] * v[1] + v[2] * v[2] + v[3] * v[3];
  }
  const float inv = 1.f / sqrtf(pf_block_sum(sq, scratch) / true_width + eps);
  for (int i = threadIdx.x * 4; i < D; i += kPfThreads * 4)
    store4(h + static_cast<size_t>(m) * D + i, *reinterpret_cast<const f32x4*>(row + i) * inv * *reinterpret_cast<const f32x4*>(weight + i));
}

// The five mixes of a token's normed input with the previous token's; the last token leaves its own for the next portion.
template <class T>
__global__ __launch_bounds__(kPfThreads) void shift_mix(const float* u, QmkHybridLayer l, int slot, int flip, int M, int rows_cap, int D, int true_width, float eps, T* out) {
  __shared__ float scratch[4];
  const int m = blockIdx.x;
  const float* row = u + static_cast<size_t>(m) * D;
  const float* prev = row - D;
  const float* before = l.shift + (static_cast<size_t>(slot) * 2 + flip) * D;
  float* after = l.shift + (static_cast<size_t>(slot) * 2 + 1 - flip) * D;
  float sq = 0.f, sp = 0.f;
  for (int i = threadIdx.x; i < D; i += kPfThreads) {
    sq = fmaf(row[i], row[i], sq);
    if (m > 0) sp = fmaf(prev[i], prev[i], sp);
  }
  const float inv = 1.f / sqrtf(pf_block_sum(sq, scratch) / true_width + eps);
  const float inv_p = 1.f / sqrtf(pf_block_sum(sp, scratch) / true_width + eps);
  for (int i = threadIdx.x * 2; i < D; i += kPfThreads * 2) {
    float h[2], d[2];
#pragma unroll
    for (int e = 0; e < 2; ++e) {
      h[e] = row[i + e] * inv * l.norm1[i + e];
      d[e] = (m > 0 ? prev[i + e] * inv_p * l.norm1[i + e] : before[i + e]) - h[e];
      if (m == M - 1) after[i + e] = h[e];
    }
#pragma unroll
    for (int q = 0; q < 5; ++q) {
      const float a = h[0] + d[0] * l.vec2[q * D + i], b = h[1] + d[1] * l.vec2[q * D + i + 1];
      T* o = out + (static_cast<size_t>(q) * rows_cap + m) * D + i;
      if constexpr (sizeof(T) == 2) *reinterpret_cast<uint32_t*>(o) = f2bf2(a, b);
      else *reinterpret_cast<float2*>(o) = make_float2(a, b);
    }
  }
}

// u[m] = causal convolution of x (zeros or the previous portion's last inputs before it), four channels a thread.
template <class T>
__global__ __launch_bounds__(kPfThreads) void causal_conv(const T* x, QmkHybridLayer l, int slot, int flip, int M, T* out) {
  const int W = l.mix_width, quads = W / 4, n = l.taps;
  const long long id = static_cast<long long>(blockIdx.x) * kPfThreads + threadIdx.x;
  if (id >= static_cast<long long>(M) * quads) return;
  const int m = static_cast<int>(id / quads), c = static_cast<int>(id % quads) * 4;
  const float* old = l.shift + (static_cast<size_t>(slot) * 2 + flip) * (n - 1) * W;
  float* now = l.shift + (static_cast<size_t>(slot) * 2 + 1 - flip) * (n - 1) * W;
  auto input = [&](int t) {   // t >= -(n - 1)
    return t >= 0 ? read4(x + static_cast<size_t>(t) * W + c) : *reinterpret_cast<const f32x4*>(old + static_cast<size_t>(t + n - 1) * W + c);
  };
  f32x4 acc = *reinterpret_cast<const f32x4*>(l.vec1 + c);
  for (int j = 0; j < n; ++j) acc += *reinterpret_cast<const f32x4*>(l.vec2 + static_cast<size_t>(j) * W + c) * input(m - (n - 1) + j);
  store4(out + static_cast<size_t>(m) * W + c, acc);
  if (m == M - 1)
    for (int j = 0; j < n - 1; ++j) *reinterpret_cast<f32x4*>(now + static_cast<size_t>(j) * W + c) = input(M - (n - 1) + j);
}

// S_t = a_t S_{t-1} + b_t, out = S y: sixteen channels a workgroup, the portion cut into 64 runs of tokens.
constexpr int kScanChannels = 16, kScanRuns = 64;
template <class T>
__global__ __launch_bounds__(kScanChannels * kScanRuns) void lru_scan(const float* a, const float* b, const T* y, QmkHybridLayer l, int slot, int M, T* out) {
  __shared__ float sa[kScanRuns][kScanChannels], sb[kScanRuns][kScanChannels];
  const int W = l.mix_width, ch = threadIdx.x % kScanChannels, run = threadIdx.x / kScanChannels;
  const int c = blockIdx.x * kScanChannels + ch;
  const int per = (M + kScanRuns - 1) / kScanRuns, lo = min(run * per, M), hi = min(lo + per, M);
  float pa = 1.f, pb = 0.f;
#pragma unroll 4
  for (int t = lo; t < hi; ++t) {
    const size_t at = static_cast<size_t>(t) * W + c;
    const float av = a[at];
    pa *= av;
    pb = fmaf(av, pb, b[at]);
  }
  sa[run][ch] = pa;
  sb[run][ch] = pb;
  __syncthreads();
  float* st = l.state + static_cast<size_t>(slot) * W + c;
  if (run == 0) {
    float s = *st;
    for (int r = 0; r < kScanRuns; ++r) {
      const float e = fmaf(sa[r][ch], s, sb[r][ch]);
      sb[r][ch] = s;      // the state the run starts from
      s = e;
    }
    *st = s;
  }
  __syncthreads();
  float s = sb[run][ch];
#pragma unroll 4
  for (int t = lo; t < hi; ++t) {
    const size_t at = static_cast<size_t>(t) * W + c;
    s = fmaf(a[at], s, b[at]);
    out[at] = from_f32<T>(s * to_f32(y[at]));
  }
}

// Keys first .. position + M - 1 side by side: new rows normed and rotated (and stored in the cache), old ones copied.
template <class T>
__global__ __launch_bounds__(kPfThreads) void latent_rows(const float* raw, QmkHybridLayer l, int slot, int first, int position, float eps, T* rows) {
  __shared__ float scratch[4];
  const int width = l.rank + l.rot_dim, pos = first + blockIdx.x;
  T* row = static_cast<T*>(l.cache) + (static_cast<size_t>(slot) * l.ring + pos % l.ring) * width;
  T* out = rows + static_cast<size_t>(blockIdx.x) * width;
  if (pos < position) {
    for (int i = threadIdx.x; i < width; i += kPfThreads) out[i] = row[i];
    return;
  }
  const float* c = raw + static_cast<size_t>(pos - position) * width;
  float sq = 0.f;
  for (int i = threadIdx.x; i < l.rank; i += kPfThreads) sq = fmaf(c[i], c[i], sq);
  const float inv = 1.f / sqrtf(pf_block_sum(sq, scratch) / l.rank_true + eps);
  for (int i = threadIdx.x * 2; i < width; i += kPfThreads * 2) {
    float a = c[i], b = c[i + 1];
    if (i < l.rank) {
      a = a * inv * l.vec0[i];
      b = b * inv * l.vec0[i + 1];
    } else {
      rotate(l, pos, i - l.rank, a, b);
    }
    row[i] = out[i] = from_f32<T>(a);
    row[i + 1] = out[i + 1] = from_f32<T>(b);
  }
}

// Keys of an attention: key j of key head h at at[j * pitch + h * head]; heads_per query heads share a key head.
template <class T>
struct Keys {
  const T* at;
  int pitch, head, heads_per;
};

// Windowed attention over expanded keys: 64 queries of one head a workgroup (16 a wave), 32 keys a step.
// Scores are computed transposed (keys x queries), so a lane holds eight weights of ONE query in exactly the shape the
// value product's second operand wants, with keys in the order 4g..4g+3, 16+4g..16+4g+3.
template <class T, int QT, int VT>   // most 32-column steps of a query, most 16-row tiles of a value
__global__ __launch_bounds__(kPfThreads) void window_attention(const T* q, Keys<T> keys, const T* rows, const T* v_t, const T* gate, QmkHybridLayer l,
                                                               int first, int position, int M, int keys_cap, T* out) {
  constexpr int kKeys = 32;
  constexpr int kPadK = 16 / sizeof(T), kPadV = 16 / sizeof(T);
  __shared__ __align__(16) T sk[kKeys][QT * 32 + kPadK];
  __shared__ __align__(16) T sv[VT * 16][kKeys + kPadV];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, g = lane >> 4, col = lane & 15;
  // Later queries see more keys where no window ends.  Workgroups 256 apart share a CU: every other such run of heads takes
  // its queries from the far end, so that a CU gets long and short ones.
  const bool mirrored = (blockIdx.y * gridDim.x >> 8 & 1) == 0;
  const int head = blockIdx.y, kv = head / keys.heads_per, q0 = (mirrored ? gridDim.x - 1 - blockIdx.x : blockIdx.x) * 64;
  const int dq = l.q_stride, steps = dq / 32, vt = l.v_dim / 16, width = l.rank + l.rot_dim;
  const int m = q0 + wave * 16 + col, pos = position + m;
  Frag<T> fq[QT];
#pragma unroll
  for (int s = 0; s < QT; ++s)
    if (s < steps) fq[s] = load_frag(q + static_cast<size_t>(min(m, M - 1)) * l.heads * dq + head * dq + s * 32 + g * 8);
  f32x4 acc[VT] = {};
  float top = -INFINITY, sum = 0.f;
  const float scale = l.scale * kLog2e;
  const int lo = max(first, position + q0 + 1 - l.window);      // the first key any of the 64 queries sees
  const int hi = min(position + q0 + 64, position + M);          // behind the last one
  constexpr int kU = 16 / sizeof(T);
  // Staging: each thread has fixed places in a tile of keys and of transposed values; the next tile is in flight while
  // this one is used.
  constexpr int kKLoads = kKeys * QT * 32 / kU / kPfThreads, kVLoads = VT * 16 * kKeys / kU / kPfThreads;
  static_assert(kKLoads * kPfThreads * kU == kKeys * QT * 32 && kVLoads * kPfThreads * kU == VT * 16 * kKeys, "every thread stages the same number of units");
  const int base0 = first + ((lo - first) & ~(kKeys - 1));
  const T* k_at[kKLoads];
  int k_step[kKLoads];
  v4u rk[kKLoads], rv[kVLoads];
#pragma unroll
  for (int i = 0; i < kKLoads; ++i) {
    const int id = i * kPfThreads + tid, r = id / (QT * 32 / kU), c = id % (QT * 32 / kU) * kU, row = base0 + r - first;
    k_at[i] = nullptr;                 // columns behind the rotated part: zeros
    k_step[i] = 0;
    if (c < l.head_dim) {
      k_at[i] = keys.at + static_cast<size_t>(row) * keys.pitch + kv * keys.head + c;
      k_step[i] = kKeys * keys.pitch;
    } else if (c < l.head_dim + l.rot_dim) {
      k_at[i] = rows + static_cast<size_t>(row) * width + l.rank + c - l.head_dim;
      k_step[i] = kKeys * width;
    }
  }
  auto fetch = [&](int base) {
#pragma unroll
    for (int i = 0; i < kKLoads; ++i) {
      const int r = (i * kPfThreads + tid) / (QT * 32 / kU);
      rk[i] = v4u{0u, 0u, 0u, 0u};
      if (k_at[i] != nullptr && base + r < hi) rk[i] = *reinterpret_cast<const v4u*>(k_at[i]);
      k_at[i] = k_at[i] == nullptr ? nullptr : k_at[i] + k_step[i];
    }
#pragma unroll
    for (int i = 0; i < kVLoads; ++i) {
      const int id = i * kPfThreads + tid, r = id / (kKeys / kU), c = id % (kKeys / kU) * kU;
      rv[i] = v4u{0u, 0u, 0u, 0u};
      if (r < l.v_dim && base + c < hi) rv[i] = *reinterpret_cast<const v4u*>(v_t + static_cast<size_t>(kv * l.v_dim + r) * keys_cap + base - first + c);
      if (base + c + kU > hi) {   // keys behind the last one: whatever the buffer holds there must not enter a sum
        T* e = reinterpret_cast<T*>(&rv[i]);
#pragma unroll
        for (int j = 0; j < kU; ++j)
          if (base + c + j >= hi) e[j] = from_f32<T>(0.f);
      }
    }
  };
  fetch(base0);
  const int first_pos = position + q0 + wave * 16;       // this wave's queries: first_pos .. first_pos + 15
  for (int base = base0; base < hi; base += kKeys) {
#pragma unroll
    for (int i = 0; i < kKLoads; ++i) {
      const int id = i * kPfThreads + tid;
      *reinterpret_cast<v4u*>(&sk[id / (QT * 32 / kU)][id % (QT * 32 / kU) * kU]) = rk[i];
    }
#pragma unroll
    for (int i = 0; i < kVLoads; ++i) {
      const int id = i * kPfThreads + tid;
      *reinterpret_cast<v4u*>(&sv[id / (kKeys / kU)][id % (kKeys / kU) * kU]) = rv[i];
    }
    __syncthreads();
    if (base + kKeys < hi) fetch(base + kKeys);
    f32x4 d[2] = {};
#pragma unroll
    for (int s = 0; s < QT; ++s)
      if (s < steps) {
#pragma unroll
        for (int t = 0; t < 2; ++t) d[t] = mma(load_frag(&sk[t * 16 + col][s * 32 + g * 8]), fq[s], d[t]);
      }
    float w[8];
    float best = top;
#pragma unroll
    for (int j = 0; j < 8; ++j) w[j] = d[j >> 2][j & 3] * scale;
    if (base + kKeys - 1 > first_pos || first_pos + 15 - base >= l.window) {   // some query does not see some key
#pragma unroll
      for (int j = 0; j < 8; ++j) {
        const int key = base + (j >> 2) * 16 + g * 4 + (j & 3), dist = pos - key;
        if (dist < 0 || dist >= l.window) w[j] = -INFINITY;
      }
    }
#pragma unroll
    for (int j = 0; j < 8; ++j) best = fmaxf(best, w[j]);
    best = fmaxf(best, __shfl_xor(best, 16));
    best = fmaxf(best, __shfl_xor(best, 32));
    const float ref = best == -INFINITY ? 0.f : best;      // no key of this query yet
    const float shrink = exp2_fast(top - ref);
    float part = 0.f;
    Frag<T> fp;
#pragma unroll
    for (int j = 0; j < 8; ++j) {
      w[j] = exp2_fast(w[j] - ref);
      part += w[j];
      fp.set(j, from_f32<T>(w[j]));
    }
    sum = sum * shrink + part;
    top = best;
#pragma unroll
    for (int t = 0; t < VT; ++t)
      if (t < vt) {
        Frag<T> fv;
        const T* r = &sv[t * 16 + col][0];
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          fv.set(j, r[g * 4 + j]);
          fv.set(4 + j, r[16 + g * 4 + j]);
        }
        acc[t] = mma(fv, fp, acc[t] * shrink);
      }
    __syncthreads();
  }
  sum += __shfl_xor(sum, 16);
  sum += __shfl_xor(sum, 32);
  if (m >= M) return;
  const float inv = 1.f / sum;
  const size_t at = static_cast<size_t>(m) * l.heads * l.v_dim + head * l.v_dim;
#pragma unroll
  for (int t = 0; t < VT; ++t)
    if (t < vt) store4(out + at + t * 16 + g * 4, acc[t] * inv * read4(gate + at + t * 16 + g * 4));
}

// The wkv recurrence: one head and eight value columns a workgroup; sixteen lanes share a column, KPL neighbouring key
// rows each, in registers.  TB tokens at a time: the next block's r, k, w, v are in flight while this one runs, a block's
// outputs leave together.  Places behind the last token or key row hold r = k = 0, w = 1, which changes nothing.
constexpr int kWkvColumns = 8, kWkvThreads = 16 * kWkvColumns;
template <int KPL, int TB>
__global__ __launch_bounds__(kWkvThreads) void wkv_scan(const float* r, const float* k, const float* v, const float* w, QmkHybridLayer l, int slot, int M, float* out) {
  constexpr int kKeys = 16 * KPL, kQuads = TB * kKeys / 4 / kWkvThreads, kValueQuads = TB * kWkvColumns / 4;
  static_assert(kQuads * kWkvThreads * 4 == TB * kKeys && kValueQuads <= kWkvThreads, "every thread stages the same number of quads");
  __shared__ __align__(16) float sr[2][TB][kKeys], sk[2][TB][kKeys], sw[2][TB][kKeys], sv[2][TB][kWkvColumns], so[2][TB][kWkvColumns];
  const int n = l.head_dim, N = l.heads * n, head = blockIdx.y, v0 = blockIdx.x * kWkvColumns;
  const int tid = threadIdx.x, part = tid & 15, e = tid >> 4;
  float* st = l.state + (static_cast<size_t>(slot) * l.heads + head) * n * n + v0 + e;
  float s[KPL], u[KPL];
#pragma unroll
  for (int i = 0; i < KPL; ++i) {
    const int row = part * KPL + i;
    s[i] = row < n ? st[row * n] : 0.f;
    u[i] = row < n ? l.vec1[head * n + row] : 0.f;
  }
  f32x4 fr[kQuads], fk[kQuads], fw[kQuads], fv = {};
  auto fetch = [&](int base) {
#pragma unroll
    for (int q = 0; q < kQuads; ++q) {
      const int id = tid + q * kWkvThreads, t = base + id / (kKeys / 4), c = id % (kKeys / 4) * 4;
      const size_t at = static_cast<size_t>(t) * N + head * n + c;
      const bool real = t < M && c < n;
      fr[q] = real ? *reinterpret_cast<const f32x4*>(r + at) : f32x4{0.f, 0.f, 0.f, 0.f};
      fk[q] = real ? *reinterpret_cast<const f32x4*>(k + at) : f32x4{0.f, 0.f, 0.f, 0.f};
      fw[q] = real ? *reinterpret_cast<const f32x4*>(w + at) : f32x4{1.f, 1.f, 1.f, 1.f};
    }
    if (tid < kValueQuads) {
      const int t = base + tid / (kWkvColumns / 4);
      fv = t < M ? *reinterpret_cast<const f32x4*>(v + static_cast<size_t>(t) * N + head * n + v0 + tid % (kWkvColumns / 4) * 4) : f32x4{0.f, 0.f, 0.f, 0.f};
    }
  };
  auto stash = [&](int buf) {
#pragma unroll
    for (int q = 0; q < kQuads; ++q) {
      const int id = tid + q * kWkvThreads, t = id / (kKeys / 4), c = id % (kKeys / 4) * 4;
      *reinterpret_cast<f32x4*>(&sr[buf][t][c]) = fr[q];
      *reinterpret_cast<f32x4*>(&sk[buf][t][c]) = fk[q];
      *reinterpret_cast<f32x4*>(&sw[buf][t][c]) = fw[q];
    }
    if (tid < kValueQuads) *reinterpret_cast<f32x4*>(&sv[buf][tid / (kWkvColumns / 4)][tid % (kWkvColumns / 4) * 4]) = fv;
  };
  fetch(0);
  stash(0);
  __syncthreads();
  int buf = 0;
  for (int base = 0; base < M; base += TB, buf ^= 1) {
    if (base + TB < M) fetch(base + TB);
    // Four tokens at a time: their sums over the sixteen lanes are taken together (two steps that halve the values while
    // they pair lanes, then plain sums), and lane p of sixteen ends up with token p % 4.
    for (int t0 = 0; t0 < TB; t0 += 4) {
      float o[4];
#pragma unroll
      for (int q = 0; q < 4; ++q) {
        const int t = t0 + q;
        const float vt = sv[buf][t][e];
        o[q] = 0.f;
#pragma unroll
        for (int i = 0; i < KPL; i += 4) {
          const f32x4 r4 = *reinterpret_cast<const f32x4*>(&sr[buf][t][part * KPL + i]), k4 = *reinterpret_cast<const f32x4*>(&sk[buf][t][part * KPL + i]),
                      w4 = *reinterpret_cast<const f32x4*>(&sw[buf][t][part * KPL + i]);
#pragma unroll
          for (int j = 0; j < 4; ++j) {
            const float kv = k4[j] * vt;
            o[q] = fmaf(r4[j], fmaf(u[i + j], kv, s[i + j]), o[q]);
            s[i + j] = fmaf(w4[j], s[i + j], kv);
          }
        }
      }
      const bool b0 = part & 1, b1 = part & 2;
      const float lo = (b0 ? o[1] : o[0]) + dpp_f32<kDppQuadXor1>(0.f, b0 ? o[0] : o[1]);
      const float hi = (b0 ? o[3] : o[2]) + dpp_f32<kDppQuadXor1>(0.f, b0 ? o[2] : o[3]);
      float sum = (b1 ? hi : lo) + dpp_f32<kDppQuadXor2>(0.f, b1 ? lo : hi);
      sum += dpp_f32<0x124>(0.f, sum);        // row_ror:4
      sum += dpp_f32<0x128>(0.f, sum);        // row_ror:8
      if (part < 4) so[buf][t0 + part][e] = sum;
    }
    if (base + TB < M) stash(buf ^ 1);
    __syncthreads();
    for (int id = tid; id < TB * kWkvColumns; id += kWkvThreads) {
      const int t = id / kWkvColumns, c = id % kWkvColumns;
      if (base + t < M) out[static_cast<size_t>(base + t) * N + head * n + v0 + c] = so[buf][t][c];
    }
  }
#pragma unroll
  for (int i = 0; i < KPL; ++i) {
    const int row = part * KPL + i;
    if (row < n) st[row * n] = s[i];
  }
}

// Per-head norm, weight and gate behind the recurrence: one wave per (token, head).
template <class T>
__global__ __launch_bounds__(kPfThreads) void wkv_out(const float* o, const T* gate, QmkHybridLayer l, int M, float eps, T* out) {
  const int id = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (id >= M * l.heads) return;
  const int n = l.head_dim, m = id / l.heads, head = id % l.heads;
  const size_t at = static_cast<size_t>(m) * l.heads * n + head * n;
  float sq = 0.f;
  for (int i = lane; i < n; i += 64) sq = fmaf(o[at + i], o[at + i], sq);
  const float inv = 1.f / sqrtf(wave_sum(sq) / l.head_dim_true + eps);
  for (int i = lane; i < n; i += 64) out[at + i] = from_f32<T>(o[at + i] * inv * l.vec0[head * n + i] * to_f32(gate[at + i]));
}

__global__ __launch_bounds__(kPfThreads) void sum_streams(const float* x, int S, int D, float* out) {
  const int m = blockIdx.x;
  for (int i = threadIdx.x; i < D; i += kPfThreads) {
    float t = 0.f;
    for (int s = 0; s < S; ++s) t += x[(static_cast<size_t>(m) * S + s) * D + i];
    out[static_cast<size_t>(m) * D + i] = t;
  }
}

}  // namespace hybrid
}  // namespace qmk
