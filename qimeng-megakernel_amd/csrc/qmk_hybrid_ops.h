// Decode ops of the hybrid route: one workgroup executes one instruction of the tensor built by
// decode_schedule_hybrid/instructions/scheduler.py.
//
// A step is a chain of stages; an instruction waits until every instruction of the stage before its own has arrived
// (all-to-all edges on the per-XCD counters of qmk_device.h), so a buffer written in one stage may be overwritten two
// stages later.  Activations between stages are fp32 and travel with device-coherent loads and stores; weights are
// streamed once, bf16, and multiplied in fp32.  What does not depend on this step's earlier stages is asked for before an
// instruction waits: its first weight rows, norm weights, recurrent states, old cache rows, the streams it will update.
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
constexpr int kMaxOutRows = kThreads / kMaxStreams;   // ... of OP_OUT_PROJECT: a thread per row and stream
constexpr int kChunk = kWaveSize * 8;         // columns one wave covers with one 16-byte load per lane
constexpr int kMaxK = 24576;                  // longest activation vector
constexpr int kAttendFloats = 33792;          // LDS of the attention op: query, key tile, scores
constexpr int kMaxRank = 512;
constexpr int kMaxHeadDim = 256;              // wkv
constexpr int kMaxParts = 64;
constexpr int kDepth = 8;                     // weight rows a wave keeps in flight and reduces together
constexpr int kAhead = 2;                     // quads of a vector a thread holds in registers (4096 elements a workgroup)
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
  int32_t next_layer;
  int32_t ctl[4];          // [0] wait result, [1] last to retire
  uint64_t t_wait;
  uint64_t stamps[4];      // timeline only: requests made, vector in LDS, rows multiplied, results stored
  float best_val;
  int32_t best_idx;
};

// The layer table never changes during a launch: read through the constant address space its fields are scalar loads
// that stay valid across barriers.
using LayerRef = const __attribute__((address_space(4))) QmkHybridLayer;
using ConstFloat = const __attribute__((address_space(4))) float;
__device__ __forceinline__ LayerRef& layer_of(const DecodeParams& p, int layer) { return ((LayerRef*)p.layers)[layer]; }

struct Op {                // decoded instruction
  int next_layer;          // the instruction behind it: its layer's table entry is fetched during the wait
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

__device__ __forceinline__ void stamp(const DecodeParams& p, Smem& s, int which) {
  if (p.timeline != nullptr && threadIdx.x == 0) s.stamps[which] = wall_clock64();
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
  } else if (threadIdx.x < 2 * kWaveSize) {
    const auto* line = (const __attribute__((address_space(4))) int32_t*)(p.layers + o.next_layer);
#pragma unroll
    for (int i = 0; i < static_cast<int>(sizeof(QmkHybridLayer) / 64); ++i) {
      const int32_t v = line[i * 16];
      asm volatile("" ::"s"(v));
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

// exp(z) as one hardware 2^x, relative error |z| 2^-24: for gates and activations.  Decays, which are multiplied up over
// thousands of tokens, take expf.
__device__ __forceinline__ float exp_fast(float z) { return exp2_fast(z * 1.4426950408889634f); }
__device__ __forceinline__ float sigmoid(float z) { return 1.f / (1.f + exp_fast(-z)); }
// 0.5 z (1 + tanh(t)) = z sigmoid(2 t), t = sqrt(2/pi) (z + 0.044715 z^3)
__device__ __forceinline__ float gelu_tanh(float z) { return z * sigmoid(1.5957691216057308f * (z + 0.044715f * z * z * z)); }
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

// ---- row streaming ----
// Rows [0, n) of w [., ld] times xs.  A wave owns fixed chunks of 512 columns (several waves share a chunk's rows where
// there are fewer than eight chunks, a wave takes every eighth chunk where there are more), so its eight columns of xs
// per lane sit in registers; it walks down the rows, eight in flight, and reduces eight rows' products at once.
// Narrow matrices (128 and 256 columns) are read as rows of 512: 4 or 2 neighbouring rows side by side.
struct RowStream {
  const u16* at;        // next row to load
  long long pitch;      // elements between rows
  int n, chunk, per, lanes, first, waves, total, ld;
  v4u r[kDepth];

  __device__ __forceinline__ int column(int c) const {
    const int col = c * kChunk + static_cast<int>(threadIdx.x & (kWaveSize - 1)) * 8;
    return col < total ? col : 0;      // a lane behind the last column multiplies whatever it reads by zero
  }
  __device__ __forceinline__ void start(const u16* w, int rows, int columns) {
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x / kWaveSize);
    int narrow = 0;                                          // log2 of the rows side by side
    if (columns == 128 && rows % 4 == 0) narrow = 2;
    if (columns == 256 && rows % 2 == 0) narrow = 1;
    per = 1 << narrow;
    lanes = kWaveSize >> narrow;
    ld = columns;
    total = columns << narrow;
    pitch = total;
    rows >>= narrow;
    const unsigned chunks = static_cast<unsigned>(total + kChunk - 1) / kChunk;
    const int share = chunks > 4 ? 0 : chunks > 2 ? 1 : chunks == 2 ? 2 : 3;     // log2 of the waves per chunk
    chunk = wave >> share;
    const int part = wave & ((1 << share) - 1);
    first = (rows * part) >> share;
    n = ((rows * (part + 1)) >> share) - first;
    waves = chunk < static_cast<int>(chunks) ? (chunks - chunk + kWaves - 1) / kWaves : 0;      // chunks of this wave: chunk, chunk + 8, ...
    if (waves == 0) n = 0;
    at = w + first * pitch;
    const u16* top = at + column(chunk);
#pragma unroll
    for (int j = 0; j < kDepth; ++j)
      if (j < n) r[j] = __builtin_nontemporal_load(reinterpret_cast<const v4u*>(top + j * pitch));
  }
  // part[wave][row] += sums; part must be zero, one barrier behind it.
  __device__ __forceinline__ void run(Smem& s) {
    if (n == 0) return;
    const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x / kWaveSize), lane = threadIdx.x & (kWaveSize - 1);
    float* out = s.part + wave * kMaxRows;
#pragma unroll 1
    for (int q = 0; q < waves; ++q) {
      const int c = chunk + q * kWaves;
      float x[8];
      {
        // (narrow matrices: every run of `lanes` lanes holds the same vector)
        const int k = per == 1 ? lane : (lane & (lanes - 1));
        float4 a = {0.f, 0.f, 0.f, 0.f}, b = a;
        if (c * kChunk + k * 8 < ld) {
          a = *reinterpret_cast<const float4*>(s.xs + c * kChunk + k * 4);
          b = *reinterpret_cast<const float4*>(s.xs + c * kChunk + kChunk / 2 + k * 4);
        }
        x[0] = a.x; x[1] = a.y; x[2] = a.z; x[3] = a.w;
        x[4] = b.x; x[5] = b.y; x[6] = b.z; x[7] = b.w;
      }
#pragma unroll 1
      for (int base = 0; base < n; base += kDepth) {
        // the group behind this one: further down, or the top of this wave's next chunk
        const bool more = base + kDepth < n;
        const int next_rows = more ? min(n - base - kDepth, kDepth) : (q + 1 < waves ? min(n, kDepth) : 0);
        const u16* next = more ? at + (base + kDepth) * pitch + column(c) : at + column(c + kWaves);
        float v[kDepth];
#pragma unroll
        for (int j = 0; j < kDepth; ++j) {
          const v4u w = r[j];
          float t = bf_lo(w.x) * x[0];
          t = fmaf(bf_hi(w.x), x[1], t);
          t = fmaf(bf_lo(w.y), x[2], t);
          t = fmaf(bf_hi(w.y), x[3], t);
          t = fmaf(bf_lo(w.z), x[4], t);
          t = fmaf(bf_hi(w.z), x[5], t);
          t = fmaf(bf_lo(w.w), x[6], t);
          t = fmaf(bf_hi(w.w), x[7], t);
          v[j] = t;
          if (j < next_rows) r[j] = __builtin_nontemporal_load(reinterpret_cast<const v4u*>(next + j * pitch));
        }
        const float t = reduce8(v, lane, lanes);
        const int row = base + (lane & 7);
        if ((lane & (lanes - 1)) < kDepth && row < n) {
          float* o = out + (first + row) * per + (per == 1 ? 0 : lane / lanes);
          *o = q == 0 ? t : *o + t;
        }
      }
    }
  }
  // Eight values per lane -> lane l holds the sum of value l % 8 over its run of `lanes` lanes (16, 32 or 64): three
  // steps that halve the values while they pair lanes, then plain sums.
  static __device__ __forceinline__ float reduce8(const float (&v)[kDepth], int lane, int lanes) {
    const bool b0 = lane & 1, b1 = lane & 2, b2 = lane & 4;
    float a[4], b[2];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const float keep = b0 ? v[2 * i + 1] : v[2 * i], give = b0 ? v[2 * i] : v[2 * i + 1];
      a[i] = keep + dpp_f32<kDppQuadXor1>(0.f, give);
    }
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const float keep = b1 ? a[2 * i + 1] : a[2 * i], give = b1 ? a[2 * i] : a[2 * i + 1];
      b[i] = keep + dpp_f32<kDppQuadXor2>(0.f, give);
    }
    const float keep = b2 ? b[1] : b[0], give = b2 ? b[0] : b[1];
    float t = keep + dpp_f32<0x124>(0.f, give);          // row_ror:4
    t += dpp_f32<0x128>(0.f, t);                          // row_ror:8
    if (lanes > 16) t += __shfl_xor(t, 16);
    if (lanes > 32) t += __shfl_xor(t, 32);
    return t;
  }
};

__device__ __forceinline__ void clear_part(Smem& s, int rows) {
  if (static_cast<int>(threadIdx.x) < rows)
#pragma unroll
    for (int w = 0; w < kWaves; ++w) s.part[w * kMaxRows + threadIdx.x] = 0.f;
}
__device__ __forceinline__ float row_total(const Smem& s, int row) {
  float t = 0.f;
#pragma unroll
  for (int w = 0; w < kWaves; ++w) t += s.part[w * kMaxRows + row];
  return t;
}

__device__ __forceinline__ float4 ld_shared_quad(const float* v) {
  const uint64_t a = ld_shared64(v), b = ld_shared64(v + 2);
  return make_float4(__uint_as_float(static_cast<uint32_t>(a)), __uint_as_float(static_cast<uint32_t>(a >> 32)),
                     __uint_as_float(static_cast<uint32_t>(b)), __uint_as_float(static_cast<uint32_t>(b >> 32)));
}
__device__ __forceinline__ float4& xs_quad(Smem& s, int i) { return *reinterpret_cast<float4*>(s.xs + xs_at(i)); }   // i % 4 == 0

// fp32 vector that other workgroups wrote in this launch -> xs (n a multiple of 4), four requests of a thread at a time
__device__ __forceinline__ void load_vector(Smem& s, const float* v, int n) {
  constexpr int kStep = kThreads * 4, kBatch = 4;
#pragma unroll 1
  for (int base = threadIdx.x * 4; base < n; base += kBatch * kStep) {
    float4 t[kBatch];
#pragma unroll
    for (int j = 0; j < kBatch; ++j)
      if (base + j * kStep < n) t[j] = ld_shared_quad(v + base + j * kStep);
#pragma unroll
    for (int j = 0; j < kBatch; ++j)
      if (base + j * kStep < n) xs_quad(s, base + j * kStep) = t[j];
  }
}

__device__ __forceinline__ int token_of(const DecodeParams& p) {
  const long long t = *p.token_in;
  return t < 0 || t >= p.vocab ? 0 : static_cast<int>(t);
}
__device__ __forceinline__ float weight_sum(const float* w, int n) {
  float t = 0.f;
#pragma unroll 1
  for (int i = 0; i < n; ++i) t += w[i];
  return t;
}

// A thread's quads i = 4 tid + 2048 j of a [n] vector, j < kAhead
__device__ __forceinline__ void load_ahead(float4 (&v)[kAhead], const float* from, int n) {
#pragma unroll
  for (int j = 0; j < kAhead; ++j) {
    const int i = (j * kThreads + static_cast<int>(threadIdx.x)) * 4;
    if (i < n) v[j] = *reinterpret_cast<const float4*>(from + i);
  }
}
__device__ __forceinline__ float4 times(float4 a, float4 b, float c) { return make_float4(a.x * b.x * c, a.y * b.y * c, a.z * b.z * c, a.w * b.w * c); }
__device__ __forceinline__ float square(float4 a, float t) { return fmaf(a.w, a.w, fmaf(a.z, a.z, fmaf(a.y, a.y, fmaf(a.x, a.x, t)))); }

// A quad of the sublayer input.  `first`: the embedding seen through the first layer's weights (their sum `g`).
__device__ __forceinline__ float4 input_quad(const DecodeParams& p, bool first, const u16* e, float g, int i) {
  if (!first) return ld_shared_quad(p.u + i);
  const uint2 t = *reinterpret_cast<const uint2*>(e + i);
  return make_float4(bf_lo(t.x) * g, bf_hi(t.x) * g, bf_lo(t.y) * g, bf_hi(t.y) * g);
}

// RMS norm of the sublayer input -> xs; `ahead`: the thread's first norm weights.
__device__ __forceinline__ void norm_to_xs(const DecodeParams& p, Smem& s, const float* weight, const float4 (&ahead)[kAhead], bool first, const float* hc_in) {
  const int D = p.width, tid = threadIdx.x;
  const u16* e = p.embed;
  float g = 0.f;
  if (first) {
    e += static_cast<size_t>(token_of(p)) * D;
    g = weight_sum(hc_in, p.streams);
  }
  float4 v[kAhead];
  float sq = 0.f;
#pragma unroll
  for (int j = 0; j < kAhead; ++j) {
    const int i = (j * kThreads + tid) * 4;
    v[j] = make_float4(0.f, 0.f, 0.f, 0.f);
    if (i < D) v[j] = input_quad(p, first, e, g, i);
  }
#pragma unroll
  for (int j = 0; j < kAhead; ++j) sq = square(v[j], sq);
#pragma unroll 1
  for (int i = (kAhead * kThreads + tid) * 4; i < D; i += kThreads * 4) {
    const float4 t = input_quad(p, first, e, g, i);
    sq = square(t, sq);
    xs_quad(s, i) = t;
  }
  const float inv = 1.f / sqrtf(block_sum(sq, s.scratch) / p.width_true + p.eps);
#pragma unroll
  for (int j = 0; j < kAhead; ++j) {
    const int i = (j * kThreads + tid) * 4;
    if (i < D) xs_quad(s, i) = times(v[j], ahead[j], inv);
  }
#pragma unroll 1
  for (int i = (kAhead * kThreads + tid) * 4; i < D; i += kThreads * 4)
    xs_quad(s, i) = times(xs_quad(s, i), *reinterpret_cast<const float4*>(weight + i), inv);
}

template <class Layer>
__device__ __forceinline__ void rotate(const Layer& l, int position, int d, float& a, float& b) {
  if (d >= l.rot_true) return;
  const size_t at = static_cast<size_t>(position) * (l.rot_true / 2) + (d >> 1);
  const float c = l.rope_cos[at], sn = l.rope_sin[at];
  const float x = a * c - b * sn;
  b = b * c + a * sn;
  a = x;
}

template <class T>
__device__ __forceinline__ T* cache_row(const DecodeParams& p, LayerRef& l, int position) {
  return static_cast<T*>(l.cache) + (static_cast<size_t>(p.slot) * l.ring + position % l.ring) * (l.rank + l.rot_dim);
}

// ---- the ops that stream weight rows: one body, so that the streaming code exists once ----
// rows of the matrix this instruction covers; false: an operand is out of range
struct Rows {
  const u16* w;
  int rows, columns;
};
__device__ __forceinline__ bool rows_of(const DecodeParams& p, LayerRef& l, const Op& o, Rows& g) {
  const int D = p.width;
  auto set = [&](const u16* w, long long row, int rows, int columns) {
    g.w = w + row * columns;
    g.rows = rows;
    g.columns = columns;
    return o.start >= 0 && o.count > 0 && rows <= kMaxRows;
  };
  switch (o.opcode) {
    case OP_IN_PROJECT:
      return o.sub >= 0 && o.sub < 5 && !((o.start | o.count) & 1) && o.start + o.count <= l.in_rows && set(l.in_w, o.start, o.count, D);
    case OP_LRU_STEP:
      return l.type == QMK_MIXER_RGLRU && o.sub >= 0 && o.sub < l.blocks && o.start + o.count <= l.block_dim &&
             set(l.mid_w, static_cast<long long>(o.sub) * 2 * l.block_dim + 2 * o.start, 2 * o.count, l.block_dim);
    case OP_LATENT_ABSORB:
      return l.type == QMK_MIXER_LATENT && o.sub >= 0 && o.sub < l.heads && o.start + o.count <= l.rank &&
             set(l.mid_w, static_cast<long long>(o.sub) * l.rank + o.start, o.count, l.head_dim);
    case OP_LATENT_VALUE:
      return l.type == QMK_MIXER_LATENT && o.sub >= 0 && o.sub < l.heads && o.start + o.count <= l.v_dim && o.extra > 0 &&
             o.extra <= p.max_splits && o.extra <= kMaxParts && set(l.uv_w, static_cast<long long>(o.sub) * l.v_dim + o.start, o.count, l.rank);
    case OP_WKV_STEP:
      return l.type == QMK_MIXER_WKV && o.sub >= 0 && o.sub < l.heads && l.head_dim <= kMaxHeadDim &&
             set(l.mid_w, static_cast<long long>(o.sub) * l.head_dim, l.head_dim, l.rank);
    case OP_OUT_PROJECT:
      if (o.count > kMaxOutRows) return false;
      if (o.sub == 1) return l.has_mlp && o.start + o.count <= D && set(l.down_w, o.start, o.count, l.ff);
      return o.start + o.count <= D && set(l.o_w, o.start, o.count, l.mix_width);
    case OP_UP_GATE: return l.has_mlp && o.start + o.count <= l.ff && set(l.mlp_w, 2LL * o.start, 2 * o.count, D);
    case OP_LM_HEAD: return o.start + o.count <= p.vocab_rows && set(p.head, o.start, o.count, D);
    default: return false;
  }
}

template <class T>
__device__ __forceinline__ bool op_rows(const DecodeParams& p, Smem& s, const Op& o) {
  LayerRef& l = layer_of(p, o.layer);
  Rows m;
  if (!rows_of(p, l, o, m)) return bad_operand(p, o, o.start);
  const int tid = threadIdx.x, D = p.width, S = p.streams;
  RowStream g;
  g.start(m.w, m.rows, m.columns);
  clear_part(s, m.rows);

  // Asked for ahead of the wait; what the arrays hold depends on the op.  Thread r of the workgroup owns row r.
  const int op = o.opcode, row = o.start + tid;
  const bool mine = tid < m.rows;
  const bool normed = op == OP_IN_PROJECT || op == OP_UP_GATE || op == OP_LM_HEAD;
  const bool wkv_in = op == OP_IN_PROJECT && l.type == QMK_MIXER_WKV;
  const bool first = o.layer == 0 && (op == OP_IN_PROJECT || (op == OP_OUT_PROJECT && o.sub == 0));
  const float* norm = op == OP_IN_PROJECT ? l.norm1 : op == OP_UP_GATE ? l.norm2 : p.final_norm;
  const size_t shift_copy = l.type == QMK_MIXER_WKV ? static_cast<size_t>(D) : static_cast<size_t>(l.taps - 1) * l.mix_width;
  const float* shift_old = l.shift + (static_cast<size_t>(p.slot) * 2 + p.flip) * shift_copy;
  float* shift_new = l.shift + (static_cast<size_t>(p.slot) * 2 + 1 - p.flip) * shift_copy;
  const float* mu = l.vec2 + static_cast<size_t>(o.sub) * D;
  float4 w0[kAhead], w1[kAhead], w2[kAhead];
  float a[kMaxStreams] = {}, b[kMaxStreams] = {};
  float out_weight = 0.f, next_weight = 0.f;
  float* state = nullptr;
  if (normed) {
    load_ahead(w0, norm, D);
    if (wkv_in) {
      load_ahead(w1, shift_old, D);
      load_ahead(w2, mu, D);
    } else if (op == OP_IN_PROJECT && l.type == QMK_MIXER_RGLRU && mine) {
      // Everything of the convolution but the current input; the kept inputs move up by one.
      const int W = l.mix_width, c = row - W;
      a[0] = l.in_b[row];
      if (c >= 0) {
        float acc = l.vec1[c];
#pragma unroll 1
        for (int j = 0; j < l.taps - 1; ++j) {
          const float x = shift_old[static_cast<size_t>(j) * W + c];
          acc = fmaf(l.vec2[static_cast<size_t>(j) * W + c], x, acc);
          if (j > 0) shift_new[static_cast<size_t>(j - 1) * W + c] = x;
        }
        a[1] = acc;
        a[2] = l.vec2[static_cast<size_t>(l.taps - 1) * W + c];
      }
    }
  } else if (op == OP_LRU_STEP) {
    if (mine) {   // rows (r, i) of a channel: neighbouring threads
      const int c = o.sub * l.block_dim + o.start + (tid >> 1);
      state = l.state + static_cast<size_t>(p.slot) * l.mix_width + c;
      a[0] = l.mid_b[2 * c + (tid & 1)];
      a[1] = l.vec0[c];
      a[2] = *state;
    }
  } else if (op == OP_WKV_STEP) {
    const int n = l.head_dim, groups = kThreads / n, e = tid % n, group = tid / n;
    state = l.state + (static_cast<size_t>(p.slot) * l.heads + o.sub) * n * n + e;
#pragma unroll
    for (int j = 0; j < kMaxStreams; ++j) {
      const int i = group + j * groups;
      if (group < groups && i < n) a[j] = state[i * n];
    }
    if (mine) {
      const int at = o.sub * n + tid;
      w0[0] = make_float4(l.mid_b[at], l.vec1[at], l.vec0[at], 0.f);
    }
  } else if (op == OP_OUT_PROJECT) {
    // Eight lanes per row, one per stream: all streams of the row, the stream's column of the mix, its output weight and
    // its weight in the next sublayer's input.  The streams may be read before the wait: every output projection of a
    // schedule deals the rows to the queues alike, so their last writer is this workgroup, and it has seen its stores
    // acknowledged.
    const int r = o.start + (tid >> 3), q = tid & 7;
    if ((tid >> 3) < m.rows && q < S) {
      const bool down = o.sub == 1;
      const float* hc = l.hc + (down ? S * (S + 2) : 0) + S;
      const float e = first ? bf2f(p.embed[static_cast<size_t>(token_of(p)) * D + r]) : 0.f;
#pragma unroll
      for (int f = 0; f < kMaxStreams; ++f) {
        if (f < S) {
          a[f] = first ? e : ld_shared_f32(p.x + static_cast<size_t>(f) * D + r);
          b[f] = hc[S + f * S + q];
        }
      }
      out_weight = hc[q];
      next_weight = (down ? l.next2 : l.next1)[q];
    }
  }
  stamp(p, s, 0);
  if (!wait_stage(p, s, o)) return false;

  // The activation vector.
  if (normed) {
    norm_to_xs(p, s, norm, w0, first, l.hc);
    if (wkv_in) {
      auto mix = [&](int i, float4 before, float4 m4) {
        const float4 h = xs_quad(s, i);
        if (o.extra) *reinterpret_cast<float4*>(shift_new + i) = h;
        xs_quad(s, i) = make_float4(h.x + (before.x - h.x) * m4.x, h.y + (before.y - h.y) * m4.y, h.z + (before.z - h.z) * m4.z, h.w + (before.w - h.w) * m4.w);
      };
#pragma unroll
      for (int j = 0; j < kAhead; ++j) {
        const int i = (j * kThreads + tid) * 4;
        if (i < D) mix(i, w1[j], w2[j]);
      }
#pragma unroll 1
      for (int i = (kAhead * kThreads + tid) * 4; i < D; i += kThreads * 4)
        mix(i, *reinterpret_cast<const float4*>(shift_old + i), *reinterpret_cast<const float4*>(mu + i));
    }
  } else if (op == OP_LATENT_VALUE) {   // merge the parts of this head
    const int heads16 = (l.heads + 15) & ~15, parts = o.extra;
    const float* from = p.part + static_cast<size_t>(o.sub) * l.rank;
    const int pitch = heads16 * l.rank;
    if (tid < parts) {
      const uint64_t ml = ld_shared64(p.ml + (static_cast<size_t>(tid) * heads16 + o.sub) * 2);
      s.aux[tid] = __uint_as_float(static_cast<uint32_t>(ml));
      s.aux[kMaxParts + tid] = __uint_as_float(static_cast<uint32_t>(ml >> 32));
    }
    if (mine) a[0] = ld_shared_f32(p.proj + l.heads * l.q_stride + o.sub * l.v_dim + row);
    constexpr int kBatch = 16;
    static_assert(kMaxRank <= kThreads && kMaxParts <= kWaveSize, "one thread per latent element, one lane per part");
    const bool in = tid < l.rank;
    float v[kBatch];
    const float* column = from + min(tid, l.rank - 1);
    auto request = [&](int base) {   // no branches: sixteen requests leave back to back
#pragma unroll
      for (int j = 0; j < kBatch; ++j) v[j] = ld_shared_f32(column + min(base + j, parts - 1) * pitch);
    };
    request(0);
    __syncthreads();
    if (tid < kWaveSize) {   // weights of the parts
      const float mx = tid < parts ? s.aux[tid] : -INFINITY, top = wave_max(mx);
      const float w = exp2_fast(mx - top), sum = wave_sum(tid < parts ? w * s.aux[kMaxParts + tid] : 0.f);
      s.aux[tid] = tid < parts ? w / sum : 0.f;
    }
    __syncthreads();
    float acc = 0.f;
#pragma unroll 1
    for (int base = 0; base < parts; base += kBatch) {
      if (base != 0) request(base);
#pragma unroll
      for (int j = 0; j < kBatch; ++j) acc = fmaf(s.aux[base + j], v[j], acc);
    }
    if (in) s.xs[xs_at(tid)] = acc;
  } else {
    const float* from = p.mix;
    if (op == OP_LRU_STEP) {
      if (mine && !(tid & 1)) a[3] = ld_shared_f32(p.proj + o.sub * l.block_dim + o.start + (tid >> 1));
      from = p.proj + l.mix_width + o.sub * l.block_dim;
    } else if (op == OP_LATENT_ABSORB) {
      from = p.proj + o.sub * l.q_stride;
    } else if (op == OP_WKV_STEP) {
      const int n = l.head_dim, N = l.heads * n, at = o.sub * n + tid;
      if (mine) {
        const float r = ld_shared_f32(p.proj + at), k = ld_shared_f32(p.proj + N + at), v = ld_shared_f32(p.proj + 2 * N + at);
        w0[0].w = ld_shared_f32(p.proj + 3 * N + at);
        s.aux[tid] = r;
        s.aux[kMaxHeadDim + tid] = k;
        s.aux[2 * kMaxHeadDim + tid] = v;
        s.aux[4 * kMaxHeadDim + tid] = w0[0].y;
      }
      from = p.proj + 4 * N;
    }
    load_vector(s, from, m.columns);
  }
  __syncthreads();
  stamp(p, s, 1);
  g.run(s);
  __syncthreads();
  stamp(p, s, 2);

  // What happens to the rows' sums; a pair of rows is a pair of lanes.
  float t = mine && op != OP_OUT_PROJECT ? row_total(s, tid) : 0.f;
  static_assert(kMaxRows <= kThreads && kMaxStreams == 8, "one row per thread, eight values ahead");
  if (op == OP_OUT_PROJECT) {
    const int r = tid >> 3, q = tid & 7;
    if (r < m.rows) {      // whole groups of eight lanes
      float now = out_weight * row_total(s, r);
#pragma unroll
      for (int f = 0; f < kMaxStreams; ++f) now = fmaf(b[f], a[f], now);
      const float u = group8_sum(next_weight * now);
      if (q == 0) st_shared_f32(p.u + o.start + r, u);
      if (q < S) st_shared_f32(p.x + static_cast<size_t>(q) * D + o.start + r, now);
    }
  } else if (op == OP_UP_GATE) {
    const float up = dpp_f32<kDppQuadXor1>(0.f, t);
    if (mine && !(tid & 1)) st_shared_f32(p.mix + o.start + (tid >> 1), gelu_tanh(t) * up);
  } else if (op == OP_IN_PROJECT) {
    const float pair = dpp_f32<kDppQuadXor1>(0.f, t);
    if (mine) {
      const int W = l.mix_width;
      int gate = 0;          // 1: sigmoid, 2: times sigmoid (silu), 3: gelu
      if (l.type == QMK_MIXER_RGLRU) {
        t += a[0];
        if (row < W) {
          gate = 3;
        } else {
          if (l.taps > 1) shift_new[static_cast<size_t>(l.taps - 2) * W + row - W] = t;
          t = fmaf(a[2], t, a[1]);
        }
      } else if (l.type == QMK_MIXER_LATENT) {
        const int q_rows = l.heads * l.q_stride, g_rows = l.heads * l.v_dim;
        int d = -1;
        if (row < q_rows) d = row % l.q_stride - l.head_dim;
        else if (row < q_rows + g_rows) gate = 1;
        else d = row - q_rows - g_rows - l.rank;
        if (d >= 0 && d < l.rot_true) {
          const size_t at = static_cast<size_t>(p.position) * (l.rot_true / 2) + (d >> 1);
          const float c = l.rope_cos[at], sn = l.rope_sin[at];
          t = t * c + ((tid & 1) ? pair * sn : -(pair * sn));
        }
      } else if (row >= 4 * W) {
        t = tanhf(t);
      } else if (row >= 3 * W) {
        gate = 2;
      }
      if (gate) {
        const float z = gate == 3 ? 1.5957691216057308f * (t + 0.044715f * t * t * t) : t;
        const float sg = sigmoid(z);
        t = gate == 1 ? sg : t * sg;
      }
      st_shared_f32(p.proj + row, t);
    }
  } else if (op == OP_LRU_STEP) {
    const float gate = sigmoid(t + a[0]), in_gate = dpp_f32<kDppQuadXor1>(0.f, gate);
    if (mine && !(tid & 1)) {
      const int c = o.start + (tid >> 1);
      const float log_a = gate * a[1];
      const float b = sqrtf(-expm1f(2.f * log_a)) * in_gate * s.xs[xs_at(c)];
      const float now = fmaf(expf(log_a), a[2], b);
      *state = now;
      st_shared_f32(p.mix + o.sub * l.block_dim + c, now * a[3]);
    }
  } else if (op == OP_LATENT_VALUE) {
    if (mine) st_shared_f32(p.mix + o.sub * l.v_dim + row, t * a[0]);
  } else if (op == OP_LATENT_ABSORB) {
    if (mine) st_shared_f32(p.absorbed + o.sub * l.rank + row, t);
    if (o.extra) {   // the step's cache row: normed latent, rotated key part
      const float* c = p.proj + l.heads * (l.q_stride + l.v_dim);
      const int width = l.rank + l.rot_dim;
      static_assert(kMaxRank <= kThreads, "one latent element per thread");
      const float v = tid < l.rank ? ld_shared_f32(c + tid) : 0.f;
      const float inv = 1.f / sqrtf(block_sum(v * v, s.scratch) / l.rank_true + p.eps);
      T* to = cache_row<T>(p, l, p.position);
      auto put = [&](int i, float e) {   // a pair of elements is a pair of lanes
        const float odd = dpp_f32<kDppQuadXor1>(0.f, e);
        if constexpr (sizeof(T) == 2) {
          if (i < width && !(i & 1)) st_shared32(to + i, f2bf2(e, odd));
        } else {
          if (i < width) st_shared_f32(to + i, e);
        }
      };
      put(tid < l.rank ? tid : width, tid < l.rank ? v * inv * l.vec0[tid] : 0.f);
#pragma unroll 1
      for (int base = 0; base < l.rot_dim; base += kThreads) {
        const int i = base + tid;
        put(i < l.rot_dim ? l.rank + i : width, i < l.rot_dim ? ld_shared_f32(c + l.rank + i) : 0.f);
      }
    }
  } else if (op == OP_WKV_STEP) {
    const int n = l.head_dim, groups = kThreads / n, e = tid % n, group = tid / n;
    const float *r = s.aux, *k = r + kMaxHeadDim, *v = k + kMaxHeadDim, *w = v + kMaxHeadDim, *u = w + kMaxHeadDim;
    if (mine) s.aux[3 * kMaxHeadDim + tid] = expf(-expf(t + w0[0].x));
    __syncthreads();
    if (group < groups) {
      float acc = 0.f;
      auto key_row = [&](int i, float old) {
        const float kv = k[i] * v[e];
        acc = fmaf(r[i], fmaf(u[i], kv, old), acc);
        state[i * n] = fmaf(w[i], old, kv);
      };
#pragma unroll
      for (int j = 0; j < kMaxStreams; ++j)
        if (group + j * groups < n) key_row(group + j * groups, a[j]);
#pragma unroll 1
      for (int i = group + kMaxStreams * groups; i < n; i += groups) key_row(i, state[i * n]);
      s.xs[group * n + e] = acc;
    }
    __syncthreads();
    float val = 0.f;
    if (mine) {
#pragma unroll 4
      for (int i = 0; i < groups; ++i) val += s.xs[i * n + tid];
    }
    const float sq = block_sum(val * val, s.scratch);   // storage columns behind the true head size hold zeros
    const float inv = 1.f / sqrtf(sq / l.head_dim_true + p.eps);
    if (mine) st_shared_f32(p.mix + o.sub * n + tid, val * inv * w0[0].z * w0[0].w);
  } else {   // OP_LM_HEAD
    if (mine) p.logits[row] = t;
    const bool real = mine && row < p.vocab;
    const float top = block_max(real ? t : -INFINITY, s.scratch);
    int where = wave_min_i32(real && t == top ? row : 0x7fffffff);   // smallest row among equals
    int* slots = reinterpret_cast<int*>(s.aux);
    if ((tid & (kWaveSize - 1)) == 0) slots[tid / kWaveSize] = where;
    __syncthreads();
    if (tid == 0) {
#pragma unroll 1
      for (int w = 1; w < kWaves; ++w) where = min(where, slots[w]);
      if (where != 0x7fffffff && (top > s.best_val || s.best_idx == 0x7fffffff)) {
        s.best_val = top;
        s.best_idx = where;
      }
    }
  }
  stamp(p, s, 3);
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

constexpr float kLog2e = 1.4426950408889634f;

// Keys of one tile of OP_LATENT_ATTEND, and the LDS floats it needs for this cache row width (host and device).
__host__ __device__ constexpr int attend_keys(int element_bytes) { return element_bytes == 2 ? 64 : 32; }
__host__ __device__ constexpr int attend_floats(int row_elements, int element_bytes) {
  const int stride = (row_elements + 31) / 32 * 32 + 8, keys = attend_keys(element_bytes), slices = kWaves / (keys / 16);
  return (16 + keys) * stride * element_bytes / 4 + slices * keys * 16 + keys * 16 + 16 * (keys + 8) + 16;
}

// Part `start` of `count` of the visible keys, heads [16 sub, 16 sub + 16).  Scores: matrix tiles of 16 keys x 16 heads,
// the row's columns split over the waves of a tile; then the weights and the running sums of weight x latent, of which an
// instruction keeps columns [128 extra, 128 extra + 128), sixteen a wave.
template <class T>
__device__ __forceinline__ bool op_latent_attend(const DecodeParams& p, Smem& s, const Op& o) {
  constexpr int kKeys = attend_keys(sizeof(T)), kTiles = kKeys / 16, kSlices = kWaves / kTiles, kPer = kKeys * 16 / kThreads, kSp = kKeys + 8;
  constexpr int kUnit = 16 / sizeof(T);
  LayerRef& l = layer_of(p, o.layer);
  const int heads16 = (l.heads + 15) & ~15;
  if (l.type != QMK_MIXER_LATENT || o.sub < 0 || o.sub * 16 >= l.heads || o.start < 0 || o.count <= 0 || o.count > p.max_splits || o.start >= o.count ||
      o.extra < 0 || o.extra * 16 * kWaves >= l.rank)
    return bad_operand(p, o, o.start);
  const int tid = threadIdx.x, lane = tid & (kWaveSize - 1), wave = __builtin_amdgcn_readfirstlane(tid / kWaveSize);
  const int width = l.rank + l.rot_dim, width32 = (width + 31) & ~31, stride = width32 + 8;
  T* sq = reinterpret_cast<T*>(s.attend);
  T* sc = sq + 16 * stride;
  float* sred = reinterpret_cast<float*>(sc + kKeys * stride);   // [slice][key][16]
  float* ss = sred + kSlices * kKeys * 16;                        // [key][16]
  T* sp = reinterpret_cast<T*>(ss + kKeys * 16);                  // [16][kSp]
  float* sa = ss + kKeys * 16 + 16 * kSp;                         // [16]

  const int first = p.position + 1 > l.window ? p.position + 1 - l.window : 0, visible = p.position + 1 - first;
  const int per = ((visible + o.count - 1) / o.count + 31) & ~31;
  const int lo = first + o.start * per, hi = min(lo + per, p.position + 1);
  const int units = width32 / kUnit;
  const int rows = l.ring, offset = p.slot * rows;
  const T* cache = static_cast<const T*>(l.cache);
  // Rows base .. base + kKeys - 1 -> sc, but for the row another workgroup of this launch appends.  (A part is never
  // longer than the ring, so a position wraps at most once.)
  auto load_tile = [&](int base) {
    constexpr int kBatch = 4;
    const int at0 = base % rows;
#pragma unroll 1
    for (int r0 = wave; r0 < kKeys; r0 += kBatch * kWaves) {
#pragma unroll 1
      for (int c = lane; c < units; c += kWaveSize) {
        v4u v[kBatch];
#pragma unroll
        for (int j = 0; j < kBatch; ++j) {
          const int r = r0 + j * kWaves, at = at0 + r >= rows ? at0 + r - rows : at0 + r;
          v[j] = v4u{0u, 0u, 0u, 0u};
          if (base + r < hi && base + r != p.position && c * kUnit < width)
            v[j] = *reinterpret_cast<const v4u*>(cache + static_cast<size_t>(offset + at) * width + c * kUnit);
        }
#pragma unroll
        for (int j = 0; j < kBatch; ++j) *reinterpret_cast<v4u*>(sc + (r0 + j * kWaves) * stride + c * kUnit) = v[j];
      }
    }
  };
  // The appended row, where this part holds it (it is then the part's last).
  auto load_appended = [&](int base) {
    if (p.position >= hi || p.position < base || p.position >= base + kKeys) return;
    const T* row = cache + static_cast<size_t>(offset + p.position % rows) * width;
#pragma unroll 1
    for (int c = tid; c * kUnit < width; c += kThreads) *reinterpret_cast<v4u*>(sc + (p.position - base) * stride + c * kUnit) = ld_shared128(row + c * kUnit);
  };
  if (lo < hi) load_tile(lo);
  stamp(p, s, 0);
  if (!wait_stage(p, s, o)) return false;
  if (lo < hi) {
    const int heads = min(16, l.heads - o.sub * 16);
#pragma unroll 1
    for (int k = tid * 2; k < width32; k += kThreads * 2) {
      uint64_t v[16];
      const float* from = k < l.rank ? p.absorbed + o.sub * 16 * l.rank + k : p.proj + o.sub * 16 * l.q_stride + l.head_dim + k - l.rank;
      const int pitch = k < l.rank ? l.rank : l.q_stride;
#pragma unroll
      for (int h = 0; h < 16; ++h) v[h] = h < heads && k < width ? ld_shared64(from + h * pitch) : 0;
#pragma unroll
      for (int h = 0; h < 16; ++h) {
        sq[h * stride + k] = from_f32<T>(__uint_as_float(static_cast<uint32_t>(v[h])));
        sq[h * stride + k + 1] = from_f32<T>(__uint_as_float(static_cast<uint32_t>(v[h] >> 32)));
      }
    }
    __syncthreads();     // the tile's row that load_appended fills has been zeroed
    load_appended(lo);
  }

  stamp(p, s, 1);
  const int head = tid & 15, key0 = tid >> 4;      // this thread's scores: keys key0, key0 + 32, ...
  float m = -INFINITY, lsum = 0.f;
  f32x4 acc = {};
  const int column0 = (o.extra * kWaves + wave) * 16;      // this wave's sixteen columns of the latent
  const bool columns = column0 < l.rank;
#pragma unroll 1
  for (int base = lo; base < hi; base += kKeys) {
    if (base != lo) {
      load_tile(base);
      __syncthreads();
      load_appended(base);
    }
    __syncthreads();
    {
      const int tile = wave % kTiles, slice = wave / kTiles, steps = width32 / 32;
      f32x4 d = {};
      for (int k = slice; k < steps; k += kSlices)
        d = mma(load_frag(sc + (tile * 16 + (lane & 15)) * stride + k * 32 + (lane >> 4) * 8),
                load_frag(sq + (lane & 15) * stride + k * 32 + (lane >> 4) * 8), d);
#pragma unroll
      for (int i = 0; i < 4; ++i) sred[(slice * kKeys + tile * 16 + (lane >> 4) * 4 + i) * 16 + (lane & 15)] = d[i];
    }
    __syncthreads();
    float score[kPer];
#pragma unroll
    for (int j = 0; j < kPer; ++j) {
      const int key = key0 + 32 * j;
      score[j] = -INFINITY;
      if (base + key < hi) {
        float t = 0.f;
#pragma unroll
        for (int q = 0; q < kSlices; ++q) t += sred[(q * kKeys + key) * 16 + head];
        score[j] = t * (l.scale * kLog2e);
      }
    }
    float top = score[0];
#pragma unroll
    for (int j = 1; j < kPer; ++j) top = fmaxf(top, score[j]);
    top = fmaxf(top, __shfl_xor(top, 16));
    top = fmaxf(top, __shfl_xor(top, 32));
    if (lane < 16) ss[wave * 16 + head] = top;
    __syncthreads();
    top = m;
#pragma unroll
    for (int k = 0; k < kWaves; ++k) top = fmaxf(top, ss[k * 16 + head]);
    const float shrink = exp2_fast(m - top);
    lsum *= shrink;
#pragma unroll
    for (int j = 0; j < kPer; ++j) {
      const float w = exp2_fast(score[j] - top);
      lsum += w;
      sp[head * kSp + key0 + 32 * j] = from_f32<T>(w);
    }
    m = top;
    if (key0 == 0) sa[head] = shrink;
    __syncthreads();
    if (columns) {
      acc *= sa[lane & 15];
#pragma unroll
      for (int kk = 0; kk < kKeys / 32; ++kk) {
        Frag<T> cf;
#pragma unroll
        for (int j = 0; j < 8; ++j) cf.set(j, sc[(kk * 32 + (lane >> 4) * 8 + j) * stride + column0 + (lane & 15)]);
        acc = mma(cf, load_frag(sp + (lane & 15) * kSp + kk * 32 + (lane >> 4) * 8), acc);
      }
    }
    __syncthreads();
  }
  stamp(p, s, 2);
  // Every thread of a head has the same maximum; the sums of its key columns are added up here.
  lsum += __shfl_xor(lsum, 16);
  lsum += __shfl_xor(lsum, 32);
  if (lane < 16) ss[wave * 16 + head] = lsum;
  __syncthreads();
  float* ml = p.ml + (static_cast<size_t>(o.start) * heads16 + o.sub * 16) * 2;
  if (key0 == 0 && o.extra == 0) {
    float t = 0.f;
#pragma unroll
    for (int k = 0; k < kWaves; ++k) t += ss[k * 16 + head];
    st_shared_f32(ml + head * 2, m);
    st_shared_f32(ml + head * 2 + 1, t);
  }
  if (columns) {
    uint64_t* at = reinterpret_cast<uint64_t*>(p.part + (static_cast<size_t>(o.start) * heads16 + o.sub * 16 + (lane & 15)) * l.rank + column0 + (lane >> 4) * 4);
#pragma unroll
    for (int i = 0; i < 2; ++i)
      __hip_atomic_store(at + i, (static_cast<uint64_t>(__float_as_uint(acc[2 * i + 1])) << 32) | __float_as_uint(acc[2 * i]), __ATOMIC_RELAXED,
                         __HIP_MEMORY_SCOPE_AGENT);
  }
  stamp(p, s, 3);
  arrive_stage(p, o);
  return true;
}

}  // namespace hybrid
}  // namespace qmk
