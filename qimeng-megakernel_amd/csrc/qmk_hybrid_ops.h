// Decode ops of the hybrid route: one workgroup executes one instruction of the tensor built by
// decode_schedule_hybrid/instructions/scheduler.py.
//
// A step is a chain of stages; an instruction waits until every instruction of the stage before its own has arrived
// (all-to-all edges on the per-XCD counters of qmk_device.h), so a buffer written in one stage may be overwritten two
// stages later.  Activations between stages are fp32 and travel with device-coherent loads and stores; weights are
// streamed once, bf16, and multiplied in fp32.  An instruction requests its first weight rows before it waits.
#pragma once

#include "qmk_device.h"
#include "qmk_hybrid.h"

namespace qmk {
namespace hybrid {

enum : int {
  OP_NOOP = 0,
  OP_IN_PROJECT = 1,      // norm1 + the mixer's input projections, with what can be done per output behind them
  OP_LRU_STEP = 2,        // gates of one block + the recurrence of its channels
  OP_LATENT_ABSORB = 3,   // W_uk^T q per head; its leading instruction appends the cache row
  OP_LATENT_ATTEND = 4,   // one part of the visible keys for 16 heads
  OP_LATENT_VALUE = 5,    // merge of the parts, W_uv, output gate
  OP_WKV_STEP = 6,        // decay, recurrence, per-head norm and gate of one head
  OP_OUT_PROJECT = 7,     // output (sub 0) or down (sub 1) projection + all streams of the residual
  OP_UP_GATE = 8,         // norm2 + gate/up rows + gelu
  OP_LM_HEAD = 9,         // final norm + vocabulary rows
};

constexpr int kMaxStreams = QMK_HYBRID_MAX_STREAMS;
constexpr int kMaxTaps = QMK_HYBRID_MAX_TAPS;
constexpr int kMaxRows = 512;                 // rows of one instruction
constexpr int kChunk = kWaveSize * 8;         // columns one wave covers with one 16-byte load per lane
constexpr int kMaxK = 24576;                  // longest activation vector
constexpr int kAttendFloats = 29696;          // LDS of the attention op: query, key tile, scores
constexpr int kMaxRank = 1024;
constexpr int kMaxHeadDim = 256;              // wkv
constexpr int kMaxParts = 64;
constexpr int kDepth = 8;                     // weight loads a wave keeps in flight
constexpr int kStageGroupRows = 54;           // the counter layout of one group of four stages (qmk_device.h)
constexpr int kStageGroupSlots = 48;

struct DecodeParams {
  const int32_t* instructions;
  const QmkHybridLayer* layers;
  int32_t* barriers;
  int32_t* status;
  uint64_t* timeline;
  uint64_t* candidates;
  const u16* embed;
  const u16* head;
  const float* final_norm;
  const int64_t* token_in;
  int64_t* token_out;
  float* logits;
  float* u;          // [D] input of the next sublayer before its norm
  float* x;          // [streams][D]
  float* proj;       // outputs of OP_IN_PROJECT
  float* mix;        // what the output / down projection reads
  float* absorbed;   // [heads][rank]
  float* part;       // [parts][heads16][rank] unnormalised sums
  float* ml;         // [parts][heads16][2] maximum (log2) and sum
  int32_t num_insts;
  int32_t num_layers;
  int32_t groups;
  int32_t width, width_true, streams;
  int32_t vocab, vocab_rows;
  int32_t slot, position, flip;
  int32_t max_splits;
  float eps;
  uint32_t spin_limit;
};

struct Smem {
  union {
    struct {
      float xs[kMaxK];
      float part[kWaves * kMaxRows];
    };
    float attend[kAttendFloats];
  };
  float aux[3072];
  float scratch[kWaves];
  int32_t inst[kInstWords];
  int32_t ctl[4];          // [0] wait result, [1] last to retire
  uint64_t t_wait;
  float best_val;
  int32_t best_idx;
};

struct Op {                // decoded instruction
  int index, opcode, layer, sub, start, count, wait_stage, wait_count, arrive_stage, extra;
};

// The counter helpers of qmk_device.h read these fields of the other routes' parameter block.
__device__ __forceinline__ Params counters_of(const DecodeParams& p) {
  Params c{};
  c.barriers = p.barriers;
  c.status = p.status;
  c.num_layer_barriers = kStageGroupRows;
  c.barrier_slots = kStageGroupSlots;
  c.flags = QMK_FLAG_XCD_COUNTERS;
  c.spin_limit = p.spin_limit;
  return c;
}

__device__ __forceinline__ bool bad_operand(const DecodeParams& p, const Op& o, int operand) {
  if (threadIdx.x == 0) report_error(counters_of(p), QMK_DEV_BAD_OPERAND, o.index, o.opcode, operand);
  return false;
}

__device__ __forceinline__ bool wait_stage(const DecodeParams& p, Smem& s, const Op& o) {
  if (o.wait_stage < 0) return true;
  const Params c = counters_of(p);
  if (threadIdx.x < kWaveSize) {
    const bool ok = wait_edge_xcd(c, o.wait_stage >> 2, 2 + (o.wait_stage & 3), o.wait_count, p.spin_limit);
    if (threadIdx.x == 0) {
      s.ctl[0] = ok;
      if (!ok) report_error(c, QMK_DEV_WAIT_TIMEOUT, o.index, o.opcode, o.wait_stage);
      if (p.timeline != nullptr) s.t_wait = wall_clock64();
    }
  }
  __syncthreads();
  return s.ctl[0] != 0;
}

__device__ __forceinline__ void arrive_stage(const DecodeParams& p, const Op& o) {
  release_stores();
  __syncthreads();
  if (threadIdx.x == 0 && o.arrive_stage >= 0) arrive_all(counters_of(p), o.arrive_stage >> 2, 2 + (o.arrive_stage & 3), 1);
}

__device__ __forceinline__ float sigmoid(float z) { return 1.f / (1.f + expf(-z)); }
__device__ __forceinline__ float gelu_tanh(float z) {
  return 0.5f * z * (1.f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
}
template <class T>
__device__ __forceinline__ float to_f32(T v) {
  if constexpr (sizeof(T) == 2) return bf2f(v);
  else return v;
}
template <class T>
__device__ __forceinline__ T from_f32(float v) {
  if constexpr (sizeof(T) == 2) return f2bf(v);
  else return v;
}

// Place of element k of an activation vector in LDS: a lane's eight columns of a chunk lie in two runs of four, each
// run side by side with the other lanes' (16-byte LDS reads without bank conflicts).
__device__ __forceinline__ int xs_at(int k) {
  return (k & ~(kChunk - 1)) + ((k & 4) << 6) + ((k & (kChunk - 8)) >> 1) + (k & 3);
}

// ---- row streaming: rows [0, n) of w [., ld], the chunks of all rows dealt to the waves in equal contiguous runs ----
struct RowStream {
  const u16* w;
  int ld, chunks, begin, end;
  int next_row, next_chunk;        // of the next load
  v4u r[kDepth];

  __device__ __forceinline__ v4u load() {
    const int lane = threadIdx.x & (kWaveSize - 1);
    const int col = next_chunk * kChunk + lane * 8;
    v4u v = {0u, 0u, 0u, 0u};
    if (col < ld) v = __builtin_nontemporal_load(reinterpret_cast<const v4u*>(w + static_cast<size_t>(next_row) * ld + col));
    if (++next_chunk == chunks) {
      next_chunk = 0;
      ++next_row;
    }
    return v;
  }
  __device__ __forceinline__ void start(const u16* rows, int n, int columns) {
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x / kWaveSize);
    w = rows;
    ld = columns;
    chunks = (columns + kChunk - 1) / kChunk;
    const int units = n * chunks;
    begin = units * wave / kWaves;
    end = units * (wave + 1) / kWaves;
    next_row = begin / chunks;
    next_chunk = begin - next_row * chunks;
#pragma unroll
    for (int j = 0; j < kDepth; ++j)
      if (begin + j < end) r[j] = load();
  }
  // Sums of the rows' products with xs into part[wave][row]; part must be zero, one barrier behind it.
  __device__ __forceinline__ void run(Smem& s) {
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x / kWaveSize), lane = threadIdx.x & (kWaveSize - 1);
    int row = begin / chunks, chunk = begin - row * chunks;
    float acc = 0.f;
    for (int base = begin; base < end; base += kDepth) {
#pragma unroll
      for (int j = 0; j < kDepth; ++j) {
        if (base + j < end) {
          if (chunk * kChunk + lane * 8 < ld) {
            const float4 a = *reinterpret_cast<const float4*>(s.xs + chunk * kChunk + lane * 4);
            const float4 b = *reinterpret_cast<const float4*>(s.xs + chunk * kChunk + kChunk / 2 + lane * 4);
            const v4u v = r[j];
            acc = fmaf(bf_lo(v.x), a.x, acc);
            acc = fmaf(bf_hi(v.x), a.y, acc);
            acc = fmaf(bf_lo(v.y), a.z, acc);
            acc = fmaf(bf_hi(v.y), a.w, acc);
            acc = fmaf(bf_lo(v.z), b.x, acc);
            acc = fmaf(bf_hi(v.z), b.y, acc);
            acc = fmaf(bf_lo(v.w), b.z, acc);
            acc = fmaf(bf_hi(v.w), b.w, acc);
          }
          if (base + j + kDepth < end) r[j] = load();
          if (++chunk == chunks || base + j + 1 == end) {
            acc = wave_sum(acc);
            if (lane == 0) s.part[wave * kMaxRows + row] = acc;
            acc = 0.f;
            if (chunk == chunks) {
              chunk = 0;
              ++row;
            }
          }
        }
      }
    }
  }
};

__device__ __forceinline__ void clear_part(Smem& s, int rows) {
  for (int i = threadIdx.x; i < rows; i += kThreads)
#pragma unroll
    for (int w = 0; w < kWaves; ++w) s.part[w * kMaxRows + i] = 0.f;
}
__device__ __forceinline__ float row_total(const Smem& s, int row) {
  float t = 0.f;
#pragma unroll
  for (int w = 0; w < kWaves; ++w) t += s.part[w * kMaxRows + row];
  return t;
}

// fp32 vector that other workgroups wrote in this launch -> xs (n even)
__device__ __forceinline__ void load_vector(Smem& s, const float* v, int n) {
  for (int i = threadIdx.x * 2; i < n; i += kThreads * 2) {
    const uint64_t t = ld_shared64(v + i);
    s.xs[xs_at(i)] = __uint_as_float(static_cast<uint32_t>(t));
    s.xs[xs_at(i + 1)] = __uint_as_float(static_cast<uint32_t>(t >> 32));
  }
}

__device__ __forceinline__ int token_of(const DecodeParams& p) {
  const long long t = *p.token_in;
  return t < 0 || t >= p.vocab ? 0 : static_cast<int>(t);
}
__device__ __forceinline__ float weight_sum(const float* w, int n) {
  float t = 0.f;
  for (int i = 0; i < n; ++i) t += w[i];
  return t;
}

// RMS norm of the sublayer input -> xs.  `first`: the input is the embedding seen through the first layer's weights.
__device__ __forceinline__ void norm_to_xs(const DecodeParams& p, Smem& s, const float* weight, bool first, const float* hc_in) {
  const int D = p.width;
  float sq = 0.f;
  if (first) {
    const u16* e = p.embed + static_cast<size_t>(token_of(p)) * D;
    const float g = weight_sum(hc_in, p.streams);
    for (int i = threadIdx.x; i < D; i += kThreads) {
      const float v = bf2f(e[i]) * g;
      sq = fmaf(v, v, sq);
      s.xs[xs_at(i)] = v;
    }
  } else {
    for (int i = threadIdx.x * 2; i < D; i += kThreads * 2) {
      const uint64_t t = ld_shared64(p.u + i);
      const float a = __uint_as_float(static_cast<uint32_t>(t)), b = __uint_as_float(static_cast<uint32_t>(t >> 32));
      sq = fmaf(a, a, sq);
      sq = fmaf(b, b, sq);
      s.xs[xs_at(i)] = a;
      s.xs[xs_at(i + 1)] = b;
    }
  }
  const float inv = 1.f / sqrtf(block_sum(sq, s.scratch) / p.width_true + p.eps);
  for (int i = threadIdx.x; i < D; i += kThreads) {
    const int k = xs_at(i);
    s.xs[k] = s.xs[k] * inv * weight[i];
  }
}

__device__ __forceinline__ const float* rope_row(const float* table, const QmkHybridLayer& l, int position) {
  return table + static_cast<size_t>(position) * (l.rot_true / 2);
}
__device__ __forceinline__ void rotate(const QmkHybridLayer& l, int position, int d, float& a, float& b) {
  if (d >= l.rot_true) return;
  const float c = rope_row(l.rope_cos, l, position)[d >> 1], sn = rope_row(l.rope_sin, l, position)[d >> 1];
  const float x = a * c - b * sn;
  b = b * c + a * sn;
  a = x;
}

__device__ __forceinline__ bool op_in_project(const DecodeParams& p, Smem& s, const Op& o) {
  const QmkHybridLayer& l = p.layers[o.layer];
  if (o.start < 0 || o.count <= 0 || o.count > kMaxRows || o.start + o.count > l.in_rows || ((o.start | o.count) & 1))
    return bad_operand(p, o, o.start);
  RowStream g;
  g.start(l.in_w + static_cast<size_t>(o.start) * p.width, o.count, p.width);
  clear_part(s, o.count);
  if (!wait_stage(p, s, o)) return false;
  norm_to_xs(p, s, l.norm1, o.layer == 0, l.hc);
  if (l.type == QMK_MIXER_WKV) {
    const size_t n = p.width, at = static_cast<size_t>(p.slot) * 2 * n;
    const float* before = l.shift + at + p.flip * n;
    float* after = l.shift + at + (1 - p.flip) * n;
    const float* mu = l.vec2 + o.sub * n;
    for (int i = threadIdx.x; i < p.width; i += kThreads) {
      const int k = xs_at(i);
      const float h = s.xs[k];
      if (o.extra) after[i] = h;
      s.xs[k] = h + (before[i] - h) * mu[i];
    }
  }
  __syncthreads();
  g.run(s);
  __syncthreads();
  for (int i = threadIdx.x * 2; i < o.count; i += kThreads * 2) {
    const int row = o.start + i;
    float a = row_total(s, i), b = row_total(s, i + 1);
    if (l.type == QMK_MIXER_RGLRU) {
      a += l.in_b[row];
      b += l.in_b[row + 1];
      const int W = l.mix_width;
      if (row < W) {
        a = gelu_tanh(a);
        b = gelu_tanh(b);
      } else {
        const size_t copy = static_cast<size_t>(l.taps - 1) * W;
        const float* old = l.shift + (static_cast<size_t>(p.slot) * 2 + p.flip) * copy;
        float* now = l.shift + (static_cast<size_t>(p.slot) * 2 + 1 - p.flip) * copy;
        float v[2] = {a, b};
#pragma unroll
        for (int e = 0; e < 2; ++e) {
          const int c = row - W + e;
          float acc = l.vec1[c];
          for (int j = 0; j < l.taps - 1; ++j) {
            const float x = old[static_cast<size_t>(j) * W + c];
            acc = fmaf(l.vec2[static_cast<size_t>(j) * W + c], x, acc);
            if (j > 0) now[static_cast<size_t>(j - 1) * W + c] = x;
          }
          if (l.taps > 1) now[static_cast<size_t>(l.taps - 2) * W + c] = v[e];
          v[e] = fmaf(l.vec2[static_cast<size_t>(l.taps - 1) * W + c], v[e], acc);
        }
        a = v[0];
        b = v[1];
      }
    } else if (l.type == QMK_MIXER_LATENT) {
      const int q_rows = l.heads * l.q_stride, g_rows = l.heads * l.v_dim;
      if (row < q_rows) {
        const int d = row % l.q_stride - l.head_dim;
        if (d >= 0) rotate(l, p.position, d, a, b);
      } else if (row < q_rows + g_rows) {
        a = sigmoid(a);
        b = sigmoid(b);
      } else {
        const int d = row - q_rows - g_rows - l.rank;
        if (d >= 0) rotate(l, p.position, d, a, b);
      }
    } else {
      const int n = l.heads * l.head_dim;
      if (row >= 4 * n) {
        a = tanhf(a);
        b = tanhf(b);
      } else if (row >= 3 * n) {
        a *= sigmoid(a);
        b *= sigmoid(b);
      }
    }
    st_shared_f32(p.proj + row, a);
    st_shared_f32(p.proj + row + 1, b);
  }
  arrive_stage(p, o);
  return true;
}

__device__ __forceinline__ bool op_lru_step(const DecodeParams& p, Smem& s, const Op& o) {
  const QmkHybridLayer& l = p.layers[o.layer];
  const int n = l.block_dim;
  if (l.type != QMK_MIXER_RGLRU || o.sub < 0 || o.sub >= l.blocks || o.start < 0 || o.count <= 0 || 2 * o.count > kMaxRows || o.start + o.count > n)
    return bad_operand(p, o, o.start);
  RowStream g;
  g.start(l.mid_w + (static_cast<size_t>(o.sub) * 2 * n + 2 * o.start) * n, 2 * o.count, n);
  clear_part(s, 2 * o.count);
  if (!wait_stage(p, s, o)) return false;
  load_vector(s, p.proj + l.mix_width + o.sub * n, n);
  __syncthreads();
  g.run(s);
  __syncthreads();
  for (int i = threadIdx.x; i < o.count; i += kThreads) {
    const int in_block = o.start + i, c = o.sub * n + in_block;
    const float r = sigmoid(row_total(s, 2 * i) + l.mid_b[2 * c]);
    const float gate = sigmoid(row_total(s, 2 * i + 1) + l.mid_b[2 * c + 1]);
    const float log_a = r * l.vec0[c];
    const float b = sqrtf(-expm1f(2.f * log_a)) * gate * s.xs[xs_at(in_block)];
    float* st = l.state + static_cast<size_t>(p.slot) * l.mix_width + c;
    const float now = fmaf(expf(log_a), *st, b);
    *st = now;
    st_shared_f32(p.mix + c, now * ld_shared_f32(p.proj + c));
  }
  arrive_stage(p, o);
  return true;
}

template <class T>
__device__ __forceinline__ T* cache_row(const DecodeParams& p, const QmkHybridLayer& l, int position) {
  return static_cast<T*>(l.cache) + (static_cast<size_t>(p.slot) * l.ring + position % l.ring) * (l.rank + l.rot_dim);
}

template <class T>
__device__ __forceinline__ bool op_latent_absorb(const DecodeParams& p, Smem& s, const Op& o) {
  const QmkHybridLayer& l = p.layers[o.layer];
  if (l.type != QMK_MIXER_LATENT || o.sub < 0 || o.sub >= l.heads || o.start < 0 || o.count <= 0 || o.count > kMaxRows || o.start + o.count > l.rank)
    return bad_operand(p, o, o.start);
  RowStream g;
  g.start(l.mid_w + (static_cast<size_t>(o.sub) * l.rank + o.start) * l.head_dim, o.count, l.head_dim);
  clear_part(s, o.count);
  if (!wait_stage(p, s, o)) return false;
  load_vector(s, p.proj + o.sub * l.q_stride, l.head_dim);
  __syncthreads();
  g.run(s);
  __syncthreads();
  for (int i = threadIdx.x; i < o.count; i += kThreads) st_shared_f32(p.absorbed + o.sub * l.rank + o.start + i, row_total(s, i));
  if (o.extra) {   // the step's cache row: normed latent, rotated key part
    const float* c = p.proj + l.heads * (l.q_stride + l.v_dim);
    float sq = 0.f;
    for (int i = threadIdx.x; i < l.rank; i += kThreads) {
      const float v = ld_shared_f32(c + i);
      sq = fmaf(v, v, sq);
    }
    const float inv = 1.f / sqrtf(block_sum(sq, s.scratch) / l.rank_true + p.eps);
    T* row = cache_row<T>(p, l, p.position);
    for (int i = threadIdx.x * 2; i < l.rank + l.rot_dim; i += kThreads * 2) {
      float a = ld_shared_f32(c + i), b = ld_shared_f32(c + i + 1);
      if (i < l.rank) {
        a = a * inv * l.vec0[i];
        b = b * inv * l.vec0[i + 1];
      }
      if constexpr (sizeof(T) == 2) {
        st_shared32(row + i, f2bf2(a, b));
      } else {
        st_shared_f32(row + i, a);
        st_shared_f32(row + i + 1, b);
      }
    }
  }
  arrive_stage(p, o);
  return true;
}

// ---- matrix-core fragments: eight consecutive k per lane, for both element types.  An fp32 product of 32 k is eight
// 16x16x4 instructions, the j-th taking every lane's j-th element: the order of k is the same permutation on both sides.
typedef float f32x4 __attribute__((ext_vector_type(4)));
template <class T>
struct Frag;
template <>
struct Frag<u16> {
  bf16x8_t v;
  __device__ __forceinline__ void set(int j, u16 e) { v[j] = __builtin_bit_cast(__bf16, e); }
};
template <>
struct Frag<float> {
  float v[8];
  __device__ __forceinline__ void set(int j, float e) { v[j] = e; }
};
__device__ __forceinline__ Frag<u16> load_frag(const u16* q) { return {*reinterpret_cast<const bf16x8_t*>(q)}; }
__device__ __forceinline__ Frag<float> load_frag(const float* q) {
  Frag<float> f;
  const float4 a = reinterpret_cast<const float4*>(q)[0], b = reinterpret_cast<const float4*>(q)[1];
  f.v[0] = a.x; f.v[1] = a.y; f.v[2] = a.z; f.v[3] = a.w;
  f.v[4] = b.x; f.v[5] = b.y; f.v[6] = b.z; f.v[7] = b.w;
  return f;
}
__device__ __forceinline__ Frag<float> widen(const Frag<u16>& a) {
  Frag<float> f;
#pragma unroll
  for (int j = 0; j < 8; ++j) f.v[j] = static_cast<float>(a.v[j]);
  return f;
}
__device__ __forceinline__ Frag<float> widen(const Frag<float>& a) { return a; }
__device__ __forceinline__ f32x4 mma(const Frag<u16>& a, const Frag<u16>& b, f32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.v, b.v, c, 0, 0, 0);
}
__device__ __forceinline__ f32x4 mma(const Frag<float>& a, const Frag<float>& b, f32x4 c) {
#pragma unroll
  for (int j = 0; j < 8; ++j) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a.v[j], b.v[j], c, 0, 0, 0);
  return c;
}
__device__ __forceinline__ f32x4 mma(const Frag<u16>& a, const Frag<float>& b, f32x4 c) { return mma(widen(a), b, c); }
__device__ __forceinline__ f32x4 mma(const Frag<float>& a, const Frag<u16>& b, f32x4 c) { return mma(a, widen(b), c); }

// Sixteen bytes of a cache row: the row this launch appends was written by another workgroup.
template <class T>
__device__ __forceinline__ v4u load_cache16(const T* at, bool appended) {
  return appended ? ld_shared128(at) : *reinterpret_cast<const v4u*>(at);
}

constexpr float kLog2e = 1.4426950408889634f;

// LDS floats OP_LATENT_ATTEND needs for this cache row width and element size (host and device).
__host__ __device__ constexpr int attend_floats(int row_elements, int element_bytes) {
  const int stride = (row_elements + 31) / 32 * 32 + 8;
  return (16 + 32) * stride * element_bytes / 4 + 4 * 2 * 16 * 16 + 32 * 16 + 16 * 40 + 16;
}

// Part `start` of `count` of the visible keys, heads [16 sub, 16 sub + 16).  Scores: matrix tiles of 16 keys x 16 heads,
// the row's columns split over four waves per tile; then p and the running sums of p c, 32 keys at a time.
template <class T>
__device__ __forceinline__ bool op_latent_attend(const DecodeParams& p, Smem& s, const Op& o) {
  const QmkHybridLayer& l = p.layers[o.layer];
  const int heads16 = (l.heads + 15) & ~15;
  if (l.type != QMK_MIXER_LATENT || o.sub < 0 || o.sub * 16 >= l.heads || o.start < 0 || o.count <= 0 || o.count > p.max_splits || o.start >= o.count)
    return bad_operand(p, o, o.start);
  if (!wait_stage(p, s, o)) return false;
  const int tid = threadIdx.x, lane = tid & (kWaveSize - 1), wave = __builtin_amdgcn_readfirstlane(tid / kWaveSize);
  const int width = l.rank + l.rot_dim, width32 = (width + 31) & ~31, stride = width32 + 8;
  T* sq = reinterpret_cast<T*>(s.attend);
  T* sc = sq + 16 * stride;
  float* sred = reinterpret_cast<float*>(sc + 32 * stride);   // [4][2][16][16]
  float* ss = sred + 4 * 2 * 16 * 16;                          // [32][16]
  T* sp = reinterpret_cast<T*>(ss + 32 * 16);                  // [16][40]
  float* sa = reinterpret_cast<float*>(ss + 32 * 16 + 16 * 40);  // [16]

  for (int i = tid; i < 16 * width32; i += kThreads) {
    const int h = i / width32, k = i - h * width32, head = o.sub * 16 + h;
    float v = 0.f;
    if (head < l.heads) {
      if (k < l.rank) v = ld_shared_f32(p.absorbed + head * l.rank + k);
      else if (k < width) v = ld_shared_f32(p.proj + head * l.q_stride + l.head_dim + k - l.rank);
    }
    sq[h * stride + k] = from_f32<T>(v);
  }
  const int first = p.position + 1 > l.window ? p.position + 1 - l.window : 0, visible = p.position + 1 - first;
  const int per = ((visible + o.count - 1) / o.count + 31) & ~31;
  const int lo = first + o.start * per, hi = min(lo + per, p.position + 1);

  const int head = tid & 15, key = tid >> 4;
  float m = -INFINITY, lsum = 0.f;
  f32x4 acc[kMaxRank / 16 / kWaves] = {};
  const int tiles = l.rank / 16;
  for (int base = lo; base < hi; base += 32) {
    const int units = width32 * static_cast<int>(sizeof(T)) / 16, per_unit = 16 / static_cast<int>(sizeof(T));
    for (int i = tid; i < 32 * units; i += kThreads) {
      const int r = i / units, c = (i - r * units) * per_unit, pos = base + r;
      v4u v = {0u, 0u, 0u, 0u};
      if (pos < hi && c < width) v = load_cache16(cache_row<T>(p, l, pos) + c, pos == p.position);
      *reinterpret_cast<v4u*>(sc + r * stride + c) = v;
    }
    __syncthreads();
    {
      const int tile = wave & 1, slice = wave >> 1, steps = width32 / 32;
      f32x4 d = {};
      for (int k = slice; k < steps; k += 4)
        d = mma(load_frag(sc + (tile * 16 + (lane & 15)) * stride + k * 32 + (lane >> 4) * 8),
                load_frag(sq + (lane & 15) * stride + k * 32 + (lane >> 4) * 8), d);
#pragma unroll
      for (int i = 0; i < 4; ++i) sred[((slice * 2 + tile) * 16 + (lane >> 4) * 4 + i) * 16 + (lane & 15)] = d[i];
    }
    __syncthreads();
    float score = -INFINITY;
    if (base + key < hi) {
      score = 0.f;
#pragma unroll
      for (int q = 0; q < 4; ++q) score += sred[(q * 2 * 16 + key) * 16 + head];
      score *= l.scale * kLog2e;
    }
    ss[key * 16 + head] = score;
    __syncthreads();
    float top = m;
#pragma unroll 8
    for (int k = 0; k < 32; ++k) top = fmaxf(top, ss[k * 16 + head]);
    const float shrink = exp2_fast(m - top), w = exp2_fast(score - top);
    lsum = lsum * shrink + w;
    m = top;
    sp[head * 40 + key] = from_f32<T>(w);
    if (key == 0) sa[head] = shrink;
    __syncthreads();
    {
      const float a = sa[lane & 15];
      const auto pf = load_frag(sp + (lane & 15) * 40 + (lane >> 4) * 8);
#pragma unroll
      for (int q = 0; q < kMaxRank / 16 / kWaves; ++q) {
        const int t = q * kWaves + wave;
        if (t < tiles) {
          Frag<T> cf;
#pragma unroll
          for (int j = 0; j < 8; ++j) cf.set(j, sc[((lane >> 4) * 8 + j) * stride + t * 16 + (lane & 15)]);
          acc[q] = mma(cf, pf, acc[q] * a);
        }
      }
    }
    __syncthreads();
  }
  // Every thread of a head has the same maximum; the sums of its 32 key columns are added up here.
  ss[key * 16 + head] = lsum;
  __syncthreads();
  float* ml = p.ml + (static_cast<size_t>(o.start) * heads16 + o.sub * 16) * 2;
  if (key == 0) {
    float t = 0.f;
    for (int k = 0; k < 32; ++k) t += ss[k * 16 + head];
    st_shared_f32(ml + head * 2, m);
    st_shared_f32(ml + head * 2 + 1, t);
  }
  float* out = p.part + (static_cast<size_t>(o.start) * heads16 + o.sub * 16 + (lane & 15)) * l.rank;
#pragma unroll
  for (int q = 0; q < kMaxRank / 16 / kWaves; ++q) {
    const int t = q * kWaves + wave;
    if (t < tiles) {
#pragma unroll
      for (int i = 0; i < 4; ++i) st_shared_f32(out + t * 16 + (lane >> 4) * 4 + i, acc[q][i]);
    }
  }
  arrive_stage(p, o);
  return true;
}

__device__ __forceinline__ bool op_latent_value(const DecodeParams& p, Smem& s, const Op& o) {
  const QmkHybridLayer& l = p.layers[o.layer];
  const int heads16 = (l.heads + 15) & ~15, parts = o.extra;
  if (l.type != QMK_MIXER_LATENT || o.sub < 0 || o.sub >= l.heads || o.start < 0 || o.count <= 0 || o.count > kMaxRows ||
      o.start + o.count > l.v_dim || parts <= 0 || parts > p.max_splits || parts > kMaxParts)
    return bad_operand(p, o, o.start);
  RowStream g;
  const int row0 = o.sub * l.v_dim + o.start;
  g.start(l.uv_w + static_cast<size_t>(row0) * l.rank, o.count, l.rank);
  clear_part(s, o.count);
  if (!wait_stage(p, s, o)) return false;
  if (threadIdx.x < parts) {
    const float* ml = p.ml + (static_cast<size_t>(threadIdx.x) * heads16 + o.sub) * 2;
    s.aux[threadIdx.x] = ld_shared_f32(ml);
    s.aux[kMaxParts + threadIdx.x] = ld_shared_f32(ml + 1);
  }
  __syncthreads();
  float top = -INFINITY, total = 0.f;
  for (int i = 0; i < parts; ++i) top = fmaxf(top, s.aux[i]);
  for (int i = 0; i < parts; ++i) total += s.aux[kMaxParts + i] * exp2_fast(s.aux[i] - top);
  const float inv = 1.f / total;
  for (int k = threadIdx.x * 2; k < l.rank; k += kThreads * 2) {
    float a = 0.f, b = 0.f;
    for (int i = 0; i < parts; ++i) {
      const float w = exp2_fast(s.aux[i] - top);
      const uint64_t t = ld_shared64(p.part + (static_cast<size_t>(i) * heads16 + o.sub) * l.rank + k);
      a = fmaf(w, __uint_as_float(static_cast<uint32_t>(t)), a);
      b = fmaf(w, __uint_as_float(static_cast<uint32_t>(t >> 32)), b);
    }
    s.xs[xs_at(k)] = a * inv;
    s.xs[xs_at(k + 1)] = b * inv;
  }
  __syncthreads();
  g.run(s);
  __syncthreads();
  for (int i = threadIdx.x; i < o.count; i += kThreads)
    st_shared_f32(p.mix + row0 + i, row_total(s, i) * ld_shared_f32(p.proj + l.heads * l.q_stride + row0 + i));
  arrive_stage(p, o);
  return true;
}

__device__ __forceinline__ bool op_wkv_step(const DecodeParams& p, Smem& s, const Op& o) {
  const QmkHybridLayer& l = p.layers[o.layer];
  const int n = l.head_dim, N = l.heads * n;
  if (l.type != QMK_MIXER_WKV || o.sub < 0 || o.sub >= l.heads || n > kMaxHeadDim) return bad_operand(p, o, o.sub);
  const int tid = threadIdx.x, at = o.sub * n;
  RowStream g;
  g.start(l.mid_w + static_cast<size_t>(at) * l.rank, n, l.rank);
  clear_part(s, n);
  float* st = l.state + (static_cast<size_t>(p.slot) * l.heads + o.sub) * n * n;
  if (!wait_stage(p, s, o)) return false;
  load_vector(s, p.proj + 4 * N, l.rank);
  float *r = s.aux, *k = r + kMaxHeadDim, *v = k + kMaxHeadDim, *w = v + kMaxHeadDim, *u = w + kMaxHeadDim, *out = u + kMaxHeadDim;
  for (int i = tid; i < n; i += kThreads) {
    r[i] = ld_shared_f32(p.proj + at + i);
    k[i] = ld_shared_f32(p.proj + N + at + i);
    v[i] = ld_shared_f32(p.proj + 2 * N + at + i);
    u[i] = l.vec1[at + i];
  }
  __syncthreads();
  g.run(s);
  __syncthreads();
  for (int i = tid; i < n; i += kThreads) w[i] = expf(-expf(row_total(s, i) + l.mid_b[at + i]));
  __syncthreads();
  const int groups = kThreads / n, e = tid % n, group = tid / n;
  float acc = 0.f;
  if (group < groups) {
    for (int i = group; i < n; i += groups) {
      const float old = st[i * n + e], kv = k[i] * v[e];
      acc = fmaf(r[i], fmaf(u[i], kv, old), acc);
      st[i * n + e] = fmaf(w[i], old, kv);
    }
    s.xs[group * n + e] = acc;
  }
  __syncthreads();
  float val = 0.f;
  if (tid < n)
    for (int i = 0; i < groups; ++i) val += s.xs[i * n + tid];
  const float sq = block_sum(val * val, s.scratch);   // storage columns behind the true head size hold zeros
  const float inv = 1.f / sqrtf(sq / l.head_dim_true + p.eps);
  if (tid < n) st_shared_f32(p.mix + at + tid, val * inv * l.vec0[at + tid] * ld_shared_f32(p.proj + 3 * N + at + tid));
  (void)out;
  arrive_stage(p, o);
  return true;
}

__device__ __forceinline__ bool op_out_project(const DecodeParams& p, Smem& s, const Op& o) {
  const QmkHybridLayer& l = p.layers[o.layer];
  const bool down = o.sub == 1;
  const int S = p.streams, D = p.width, K = down ? l.ff : l.mix_width;
  if (o.start < 0 || o.count <= 0 || o.count > kMaxRows || o.start + o.count > D || (down && !l.has_mlp)) return bad_operand(p, o, o.start);
  RowStream g;
  g.start((down ? l.down_w : l.o_w) + static_cast<size_t>(o.start) * K, o.count, K);
  clear_part(s, o.count);
  // Only this instruction touches these rows of the streams in this stage, and their last writer arrived long ago.
  if (!wait_stage(p, s, o)) return false;
  load_vector(s, p.mix, K);
  __syncthreads();
  g.run(s);
  __syncthreads();
  const bool first = o.layer == 0 && !down;
  const float* hc = l.hc + (down ? S * (S + 2) : 0);
  const float* next = down ? l.next2 : l.next1;
  for (int i = threadIdx.x; i < o.count; i += kThreads) {
    const int row = o.start + i;
    const float y = row_total(s, i);
    float old[kMaxStreams];
    const float e = first ? bf2f(p.embed[static_cast<size_t>(token_of(p)) * D + row]) : 0.f;
#pragma unroll
    for (int t = 0; t < kMaxStreams; ++t) old[t] = t < S ? (first ? e : ld_shared_f32(p.x + static_cast<size_t>(t) * D + row)) : 0.f;
    float u = 0.f;
    for (int t = 0; t < S; ++t) {
      float now = hc[S + t] * y;
#pragma unroll
      for (int q = 0; q < kMaxStreams; ++q)
        if (q < S) now = fmaf(hc[2 * S + q * S + t], old[q], now);
      st_shared_f32(p.x + static_cast<size_t>(t) * D + row, now);
      u = fmaf(next[t], now, u);
    }
    st_shared_f32(p.u + row, u);
  }
  arrive_stage(p, o);
  return true;
}

__device__ __forceinline__ bool op_up_gate(const DecodeParams& p, Smem& s, const Op& o) {
  const QmkHybridLayer& l = p.layers[o.layer];
  if (!l.has_mlp || o.start < 0 || o.count <= 0 || 2 * o.count > kMaxRows || o.start + o.count > l.ff) return bad_operand(p, o, o.start);
  RowStream g;
  g.start(l.mlp_w + static_cast<size_t>(2 * o.start) * p.width, 2 * o.count, p.width);
  clear_part(s, 2 * o.count);
  if (!wait_stage(p, s, o)) return false;
  norm_to_xs(p, s, l.norm2, false, nullptr);
  __syncthreads();
  g.run(s);
  __syncthreads();
  for (int i = threadIdx.x; i < o.count; i += kThreads)
    st_shared_f32(p.mix + o.start + i, gelu_tanh(row_total(s, 2 * i)) * row_total(s, 2 * i + 1));
  arrive_stage(p, o);
  return true;
}

__device__ __forceinline__ bool op_lm_head(const DecodeParams& p, Smem& s, const Op& o) {
  if (o.start < 0 || o.count <= 0 || o.count > kMaxRows || o.start + o.count > p.vocab_rows) return bad_operand(p, o, o.start);
  RowStream g;
  g.start(p.head + static_cast<size_t>(o.start) * p.width, o.count, p.width);
  clear_part(s, o.count);
  if (!wait_stage(p, s, o)) return false;
  norm_to_xs(p, s, p.final_norm, false, nullptr);
  __syncthreads();
  g.run(s);
  __syncthreads();
  float best = -INFINITY;
  int where = 0x7fffffff;
  for (int i = threadIdx.x; i < o.count; i += kThreads) {
    const float v = row_total(s, i);
    p.logits[o.start + i] = v;
    if (o.start + i < p.vocab && (v > best || where == 0x7fffffff)) {
      best = v;
      where = o.start + i;
    }
  }
  const float top = block_max(best, s.scratch);
  // smallest row among equals
  int mine = (where != 0x7fffffff && best == top) ? where : 0x7fffffff;
  mine = wave_min_i32(mine);
  int* slots = reinterpret_cast<int*>(s.aux);
  if ((threadIdx.x & (kWaveSize - 1)) == 0) slots[threadIdx.x / kWaveSize] = mine;
  __syncthreads();
  if (threadIdx.x == 0) {
    for (int w = 1; w < kWaves; ++w) mine = min(mine, slots[w]);
    if (mine != 0x7fffffff && (top > s.best_val || s.best_idx == 0x7fffffff)) {
      s.best_val = top;
      s.best_idx = mine;
    }
  }
  arrive_stage(p, o);
  return true;
}

}  // namespace hybrid
}  // namespace qmk
