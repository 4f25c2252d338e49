// Decode ops of the hybrid route: one workgroup executes one instruction of the tensor built by
// decode_schedule_hybrid/instructions/scheduler.py.
//
// A step is a chain of stages; an instruction waits until every instruction of the stage before its own has arrived
// (all-to-all edges on the per-XCD counters of qmk_device.h), so a buffer written in one stage may be overwritten two
// stages later.  Activations between stages are fp32 and travel with device-coherent loads and stores; weights are
// streamed once, bf16, and multiplied in fp32.  On a plain residual no stage adds to it: the instructions that read it next
// add what the layer run before has left (each for itself, one of them keeps the sum), so a norm over a branch's whole
// output costs no stage of its own.  What does not depend on this step's earlier stages is asked for before an
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
  OP_ATTEND = 4,          // one part of the visible keys for 16 heads
  OP_LATENT_VALUE = 5,    // merge of the parts, W_uv, output gate
  OP_WKV_STEP = 6,        // decay, recurrence, per-head norm and gate of one head
  OP_OUT_PROJECT = 7,     // output (sub 0) or down (sub 1) projection + all streams of the residual
  OP_UP_GATE = 8,         // norm2 + gate/up rows + gelu
  OP_LM_HEAD = 9,         // final norm + vocabulary rows
  OP_STATE_STEP = 10,     // gla, delta: decays and recurrence of some value columns of one head
  OP_ATTEND_MERGE = 11,   // merge of the parts of one head, output gate
  OP_JOIN = 12,           // rows of [x; embedding] -> x
  OP_GATE = 13,           // delta: rows of the output gate
};

constexpr int kMaxStreams = QMK_HYBRID_MAX_STREAMS;
constexpr int kMaxTaps = QMK_HYBRID_MAX_TAPS;
constexpr int kMaxRows = 512;                 // rows of one instruction
constexpr int kMaxOutRows = kThreads / kMaxStreams;   // ... of OP_OUT_PROJECT: a thread per row and stream
constexpr int kChunk = kWaveSize * 8;         // columns one wave covers with one 16-byte load per lane
constexpr int kMaxK = 24576;                  // longest activation vector
constexpr int kAttendFloats = 33792;          // LDS of the attention op: query, key tile, scores
constexpr int kMaxRank = 512;
constexpr int kMaxHeadDim = 256;              // wkv, gla, delta
constexpr int kStateColumns = 64;             // value columns of one OP_STATE_STEP
constexpr int kStateRows = 32;                // key rows of the state one of its threads holds: 256 rows / (512 / 64) threads a column
constexpr int kStateBatch = 8;                // ... taken together, without branches: rows behind the last one count with weights of zero
constexpr int kStateVector = kMaxHeadDim + kStateBatch * kThreads / 16;   // places of q, k and the decays in LDS, zeros behind head_dim
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
  float* x;          // [streams][D], plain: [2][D]
  float* out;        // plain: [branches, feed-forward][D] what a layer run adds to x
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
  float eps, logit_scale, logit_softcap;
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
  float scratch[3 * kWaves];
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

// Three sums over the workgroup at once; `scratch` holds 3 kWaves floats.
__device__ __forceinline__ void block_sum3(float (&v)[3], float* scratch) {
  const int wave = threadIdx.x / kWaveSize;
#pragma unroll
  for (int i = 0; i < 3; ++i) v[i] = wave_sum(v[i]);
  __syncthreads();
  if ((threadIdx.x & (kWaveSize - 1)) == 0)
#pragma unroll
    for (int i = 0; i < 3; ++i) scratch[i * kWaves + wave] = v[i];
  __syncthreads();
#pragma unroll
  for (int i = 0; i < 3; ++i) {
    v[i] = 0.f;
#pragma unroll
    for (int w = 0; w < kWaves; ++w) v[i] += scratch[i * kWaves + w];
  }
}

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

__device__ __forceinline__ void st_shared_quad(float* to, float4 v) {
  auto pair = [](float lo, float hi) { return (static_cast<uint64_t>(__float_as_uint(hi)) << 32) | __float_as_uint(lo); };
  __hip_atomic_store(reinterpret_cast<uint64_t*>(to), pair(v.x, v.y), __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
  __hip_atomic_store(reinterpret_cast<uint64_t*>(to) + 1, pair(v.z, v.w), __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
}
__device__ __forceinline__ float4 embed_quad(const u16* e, int i) {
  const uint2 t = *reinterpret_cast<const uint2*>(e + i);
  return make_float4(bf_lo(t.x), bf_hi(t.x), bf_lo(t.y), bf_hi(t.y));
}
__device__ __forceinline__ float4 plus(float4 a, float4 b) { return make_float4(a.x + b.x, a.y + b.y, a.z + b.z, a.w + b.w); }
__device__ __forceinline__ float4 multiply_add(float4 a, float4 b, float c, float4 t) {   // a b c + t
  return make_float4(fmaf(a.x * b.x, c, t.x), fmaf(a.y * b.y, c, t.y), fmaf(a.z * b.z, c, t.z), fmaf(a.w * b.w, c, t.w));
}

// The plain residual as a run (or the model's norm, or a loop's pass) reads it: the copy `x_from` plus what the run `prev`
// left.  normed: its norm under `weight` -> xs (`ahead`: the thread's first weights); otherwise [x; embedding] -> xs.
// keep: also leaves the sum in copy `x_to`.
__device__ __forceinline__ void residual_to_xs(const DecodeParams& p, Smem& s, LayerRef& l, bool normed, bool keep, const float* weight, const float4 (&ahead)[kAhead]) {
  const int D = p.width, tid = threadIdx.x;
  const u16* e = p.embed;
  if (l.x_from < 0 || !normed) e += static_cast<size_t>(token_of(p)) * D;
  const float* x = l.x_from < 0 ? nullptr : p.x + static_cast<size_t>(l.x_from) * D;
  const bool added = l.prev >= 0;
  LayerRef& before = layer_of(p, added ? l.prev : 0);
  const bool two = added && before.branches == 2, ff = added && before.has_mlp;
  const float *wa = nullptr, *wb = nullptr;
  if (two) {
    wa = before.out_norm;
    wb = layer_of(p, l.prev + 1).out_norm;
  }
  // x, feed-forward and a lone branch in `v`; two branches in `a` and `b`, their norm weights in `na` and `nb`
  auto fetch = [&](int i, float4& v, float4& a, float4& b, float4& na, float4& nb) {
    v = x == nullptr ? embed_quad(e, i) : ld_shared_quad(x + i);
    if (!added) return;
    a = ld_shared_quad(p.out + i);
    if (two) {
      b = ld_shared_quad(p.out + D + i);
      na = *reinterpret_cast<const float4*>(wa + i);
      nb = *reinterpret_cast<const float4*>(wb + i);
    }
    if (ff) v = plus(v, ld_shared_quad(p.out + static_cast<size_t>(QMK_HYBRID_MAX_BRANCHES) * D + i));
    if (!two) v = plus(v, a);
  };
  float4 v[kAhead], a[kAhead], b[kAhead], na[kAhead], nb[kAhead];
  const float4 zero = make_float4(0.f, 0.f, 0.f, 0.f);
  float sum[3] = {0.f, 0.f, 0.f};
#pragma unroll
  for (int j = 0; j < kAhead; ++j) {
    const int i = (j * kThreads + tid) * 4;
    v[j] = a[j] = b[j] = na[j] = nb[j] = zero;
    if (i < D) fetch(i, v[j], a[j], b[j], na[j], nb[j]);
  }
  float sa = 0.f, sb = 0.f;
  if (two) {
#pragma unroll
    for (int j = 0; j < kAhead; ++j) {
      sum[0] = square(a[j], sum[0]);
      sum[1] = square(b[j], sum[1]);
    }
#pragma unroll 1
    for (int i = (kAhead * kThreads + tid) * 4; i < D; i += kThreads * 4) {
      sum[0] = square(ld_shared_quad(p.out + i), sum[0]);
      sum[1] = square(ld_shared_quad(p.out + D + i), sum[1]);
    }
    block_sum3(sum, s.scratch);
    sa = before.out_scale / sqrtf(sum[0] / p.width_true + p.eps);
    sb = before.out_scale / sqrtf(sum[1] / p.width_true + p.eps);
#pragma unroll
    for (int j = 0; j < kAhead; ++j) v[j] = multiply_add(b[j], nb[j], sb, multiply_add(a[j], na[j], sa, v[j]));
  }
  float* x_to = p.x + static_cast<size_t>(l.x_to) * D;
  float total = 0.f;
  auto take = [&](int i, float4 t) {
    total += t.x + t.y + t.z + t.w;
    if (keep) st_shared_quad(x_to + i, t);
    if (!normed) {
      xs_quad(s, i) = t;
      xs_quad(s, D + i) = embed_quad(e, i);
    }
  };
#pragma unroll
  for (int j = 0; j < kAhead; ++j) {
    const int i = (j * kThreads + tid) * 4;
    if (i < D) take(i, v[j]);
  }
#pragma unroll 1
  for (int i = (kAhead * kThreads + tid) * 4; i < D; i += kThreads * 4) {
    float4 t = zero, ta = zero, tb = zero, ua = zero, ub = zero;
    fetch(i, t, ta, tb, ua, ub);
    if (two) t = multiply_add(tb, ub, sb, multiply_add(ta, ua, sa, t));
    take(i, t);
    if (normed) xs_quad(s, i) = t;
  }
  if (!normed) return;
  const float mean = l.norm == QMK_NORM_LAYER ? block_sum(total, s.scratch) / p.width_true : 0.f;
  auto centred = [&](int i, float4 t) {   // storage columns behind the true width stay zero
    return make_float4(i < p.width_true ? t.x - mean : 0.f, i + 1 < p.width_true ? t.y - mean : 0.f, i + 2 < p.width_true ? t.z - mean : 0.f,
                       i + 3 < p.width_true ? t.w - mean : 0.f);
  };
  float sq = 0.f;
#pragma unroll
  for (int j = 0; j < kAhead; ++j) {
    v[j] = centred((j * kThreads + tid) * 4, v[j]);
    sq = square(v[j], sq);
  }
#pragma unroll 1
  for (int i = (kAhead * kThreads + tid) * 4; i < D; i += kThreads * 4) {
    const float4 t = centred(i, xs_quad(s, i));
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

// What a gla or delta entry left in xs, head by head: RMS norm over the head's values, weight, output gate.
__device__ __forceinline__ void norm_heads(const DecodeParams& p, Smem& s, LayerRef& l) {
  const int lane = threadIdx.x & (kWaveSize - 1), wave = threadIdx.x / kWaveSize, n = l.v_dim;
  const float* gate = p.proj + l.proj_at + (l.type == QMK_MIXER_DELTA ? l.in_rows : 2 * l.heads * l.head_dim + l.mix_width);
  __syncthreads();
  constexpr int kPer = kMaxHeadDim / kWaveSize;
#pragma unroll 1
  for (int head = wave; head < l.heads; head += kWaves) {
    float v[kPer], g[kPer], sq = 0.f;
#pragma unroll
    for (int j = 0; j < kPer; ++j) {
      const int i = j * kWaveSize + lane;
      v[j] = g[j] = 0.f;
      if (i < n) {
        v[j] = s.xs[xs_at(head * n + i)];
        g[j] = ld_shared_f32(gate + head * n + i) * l.vec0[i];
      }
      sq = fmaf(v[j], v[j], sq);
    }
    const float inv = 1.f / sqrtf(wave_sum(sq) / l.v_true + p.eps);
#pragma unroll
    for (int j = 0; j < kPer; ++j) {
      const int i = j * kWaveSize + lane;
      if (i < n) s.xs[xs_at(head * n + i)] = v[j] * inv * g[j];
    }
  }
}

// log(1 + e^z) and the decays of the gated recurrences
__device__ __forceinline__ float softplus(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }
template <class Layer>
__device__ __forceinline__ float delta_decay(const Layer& l, int head, float z) { return expf(l.vec1[head] * softplus(z)); }
template <class Layer>
__device__ __forceinline__ float gla_decay(const Layer& l, float z) { return expf(-softplus(-z) * l.decay_scale); }
template <class Layer>
__host__ __device__ constexpr int conv_channels(const Layer& l) { return 2 * l.kv_heads * l.head_dim + l.heads * l.v_dim; }
__device__ __forceinline__ float soft_cap(float z, float cap) { return cap > 0.f ? cap * tanhf(z / cap) : z; }

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
      if (p.streams > 0 && o.count > kMaxOutRows) return false;
      if (o.sub == 1) return l.has_mlp && o.start + o.count <= D && set(l.down_w, o.start, o.count, l.ff);
      return l.type <= QMK_MIXER_DELTA && o.start + o.count <= D && set(l.o_w, o.start, o.count, l.mix_width);
    case OP_UP_GATE: return l.has_mlp && o.start + o.count <= l.ff && set(l.mlp_w, 2LL * o.start, 2 * o.count, D);
    case OP_STATE_STEP: {
      if ((l.type != QMK_MIXER_GLA && l.type != QMK_MIXER_DELTA) || o.sub < 0 || o.sub >= l.heads || l.head_dim > kMaxHeadDim) return false;
      return o.count <= kStateColumns && o.start + o.count <= l.v_dim && set(l.mid_w, static_cast<long long>(o.sub) * l.head_dim, l.head_dim, l.rank);
    }
    case OP_GATE: return l.type == QMK_MIXER_DELTA && o.start + o.count <= l.mix_width && set(l.gate_w, o.start, o.count, l.gate_rank);
    case OP_JOIN: return l.type == QMK_ENTRY_JOIN && o.start + o.count <= D && set(l.in_w, o.start, o.count, 2 * D);
    case OP_LM_HEAD: return (p.streams > 0 || l.type == QMK_ENTRY_FINAL) && o.start + o.count <= p.vocab_rows && set(p.head, o.start, o.count, D);
    default: return false;
  }
}

// PLAIN: the kernel of a plain residual (its entries, its ops), which holds none of the other kernel's code, nor that of its.
template <class T, bool PLAIN>
__device__ __forceinline__ bool op_rows(const DecodeParams& p, Smem& s, const Op& o) {
  LayerRef& l = layer_of(p, o.layer);
  constexpr bool plain = PLAIN;
  constexpr unsigned kOps = 1u << OP_IN_PROJECT | 1u << OP_OUT_PROJECT | 1u << OP_UP_GATE | 1u << OP_LM_HEAD |
                            (plain ? 1u << OP_STATE_STEP | 1u << OP_JOIN | 1u << OP_GATE : 1u << OP_LRU_STEP | 1u << OP_LATENT_ABSORB | 1u << OP_LATENT_VALUE | 1u << OP_WKV_STEP);
  const int op = o.opcode, type = l.type;
  if (!(kOps >> op & 1)) return bad_operand(p, o, o.opcode);
  __builtin_assume(kOps >> op & 1);
  __builtin_assume(plain ? type >= QMK_MIXER_GLA : type <= QMK_MIXER_WKV);
  Rows m;
  if (!rows_of(p, l, o, m)) return bad_operand(p, o, o.start);
  const int tid = threadIdx.x, D = p.width, S = p.streams;
  LayerRef& lead = layer_of(p, o.layer - l.branch);      // the run's first entry
  RowStream g;
  g.start(m.w, m.rows, m.columns);
  clear_part(s, m.rows);

  // Asked for ahead of the wait; what the arrays hold depends on the op.  Thread r of the workgroup owns row r.
  const int row = o.start + tid;
  const bool mine = tid < m.rows;
  const bool normed = op == OP_IN_PROJECT || op == OP_UP_GATE || op == OP_LM_HEAD;
  const bool wkv_in = !plain && op == OP_IN_PROJECT && type == QMK_MIXER_WKV;
  const bool reads_x = plain && (normed || op == OP_JOIN);
  const bool first = !plain && o.layer == 0 && (op == OP_IN_PROJECT || (op == OP_OUT_PROJECT && o.sub == 0));
  const float* norm = plain ? lead.norm1 : op == OP_IN_PROJECT ? l.norm1 : op == OP_UP_GATE ? l.norm2 : p.final_norm;
  const int channels = type == QMK_MIXER_DELTA ? conv_channels(l) : l.mix_width;
  const size_t shift_copy = type == QMK_MIXER_WKV ? static_cast<size_t>(D) : static_cast<size_t>(l.taps - 1) * channels;
  const float* shift_old = l.shift + (static_cast<size_t>(p.slot) * 2 + p.flip) * shift_copy;
  float* shift_new = l.shift + (static_cast<size_t>(p.slot) * 2 + 1 - p.flip) * shift_copy;
  const float* mu = l.vec2 + static_cast<size_t>(o.sub) * D;
  float4 w0[kAhead], w1[kAhead], w2[kAhead];
  float a[kMaxStreams] = {}, b[kMaxStreams] = {};
  float out_weight = 0.f, next_weight = 0.f;
  float held[kStateRows];      // OP_STATE_STEP: this thread's rows of the state
  float* state = nullptr;
  if (normed) {
    load_ahead(w0, norm, D);
    if (wkv_in) {
      load_ahead(w1, shift_old, D);
      load_ahead(w2, mu, D);
    } else if (op == OP_IN_PROJECT && type == (plain ? QMK_MIXER_DELTA : QMK_MIXER_RGLRU) && mine) {
      // Everything of the convolution but the current input; the kept inputs move up by one.
      constexpr bool lru = !plain;
      const int W = channels, c = lru ? row - W : row;
      if (lru) a[0] = l.in_b[row];
      if (c >= 0 && c < W) {
        float acc = lru ? l.vec1[c] : 0.f;
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
  } else if (!plain && op == OP_LRU_STEP) {
    if (mine) {   // rows (r, i) of a channel: neighbouring threads
      const int c = o.sub * l.block_dim + o.start + (tid >> 1);
      state = l.state + static_cast<size_t>(p.slot) * l.mix_width + c;
      a[0] = l.mid_b[2 * c + (tid & 1)];
      a[1] = l.vec0[c];
      a[2] = *state;
    }
  } else if (!plain && op == OP_WKV_STEP) {
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
  } else if (plain && op == OP_STATE_STEP) {
    const int n = o.count, groups = kThreads / n, e = tid % n, group = tid / n;
    state = l.state + (static_cast<size_t>(p.slot) * l.heads + o.sub) * l.head_dim * l.v_dim + o.start + e;
#pragma unroll
    for (int j0 = 0; j0 < kStateRows; j0 += kStateBatch) {
      if (j0 * groups < l.head_dim) {
#pragma unroll
        for (int j = j0; j < j0 + kStateBatch; ++j) held[j] = state[static_cast<size_t>(min(group + j * groups, l.head_dim - 1)) * l.v_dim];
      }
    }
    static_assert(3 * kStateVector + kStateColumns <= 3072 && kStateVector <= 2 * kThreads, "q, k, decays and values in aux");
#pragma unroll
    for (int i = 0; i < 3; ++i)
      for (int at = l.head_dim + tid; at < kStateVector; at += kThreads) s.aux[i * kStateVector + at] = 0.f;
    if (mine) a[0] = l.mid_b[o.sub * l.head_dim + tid];
  } else if (op == OP_OUT_PROJECT && !plain) {
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
  if (plain && reads_x) {
    residual_to_xs(p, s, lead, normed, op == OP_IN_PROJECT && o.extra, norm, w0);
  } else if (normed) {
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
  } else if (!plain && op == OP_LATENT_VALUE) {   // merge the parts of this head
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
    const float* from = p.mix + (op == OP_OUT_PROJECT && o.sub == 1 ? l.ff_at : l.mix_at);
    if (plain && op == OP_STATE_STEP) {
      // query, key (unit vectors for the delta rule) and values of the head
      const bool delta = type == QMK_MIXER_DELTA;
      const int n = l.v_dim, dim = l.head_dim, keys = l.kv_heads * dim, kv = o.sub / (l.heads / l.kv_heads);
      const float* proj = p.proj + l.proj_at;
      float q = 0.f, k = 0.f;
      if (tid < dim) {
        q = ld_shared_f32(proj + kv * dim + tid);
        k = ld_shared_f32(proj + keys + kv * dim + tid);
      }
      if (tid < o.count) s.aux[3 * kStateVector + tid] = ld_shared_f32(proj + 2 * keys + o.sub * n + o.start + tid);
      from = proj + 2 * keys + l.heads * n * (delta ? 1 : 2);
      if (delta) a[3] = ld_shared_f32(from + l.rank + l.gate_rank + o.sub);      // beta
      if (!delta) q *= l.q_scale;                       // (the projection is left unscaled)
      float dots[3] = {q * q, k * k, q * k};
      block_sum3(dots, s.scratch);
      if (delta) {
        const float iq = l.q_scale / sqrtf(dots[0] + 1e-6f), ik = 1.f / sqrtf(dots[1] + 1e-6f);
        q *= iq;
        k *= ik;
        dots[2] *= iq * ik;
      }
      a[4] = dots[2];
      if (tid < dim) {
        s.aux[tid] = q;
        s.aux[kStateVector + tid] = k;
      }
    } else if (plain && op == OP_GATE) {
      from = p.proj + l.proj_at + conv_channels(l) + l.rank;
    } else if (!plain && op == OP_LRU_STEP) {
      if (mine && !(tid & 1)) a[3] = ld_shared_f32(p.proj + o.sub * l.block_dim + o.start + (tid >> 1));
      from = p.proj + l.mix_width + o.sub * l.block_dim;
    } else if (!plain && op == OP_LATENT_ABSORB) {
      from = p.proj + o.sub * l.q_stride;
    } else if (!plain && op == OP_WKV_STEP) {
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
    if (plain && op == OP_OUT_PROJECT && o.sub == 0 && l.type != QMK_MIXER_ATTENTION) norm_heads(p, s, l);
  }
  __syncthreads();
  stamp(p, s, 1);
  g.run(s);
  __syncthreads();
  stamp(p, s, 2);

  // What happens to the rows' sums; a pair of rows is a pair of lanes.
  float t = mine && (plain || op != OP_OUT_PROJECT) ? row_total(s, tid) : 0.f;
  static_assert(kMaxRows <= kThreads && kMaxStreams == 8, "one row per thread, eight values ahead");
  if (plain && op == OP_JOIN) {
    if (mine) st_shared_f32(p.x + static_cast<size_t>(l.x_to) * D + row, t);
  } else if (op == OP_OUT_PROJECT && plain) {
    if (mine) st_shared_f32(p.out + static_cast<size_t>(o.sub == 1 ? QMK_HYBRID_MAX_BRANCHES : l.branch) * D + row, t);
  } else if (op == OP_OUT_PROJECT) {
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
    if (mine && !(tid & 1)) st_shared_f32(p.mix + l.ff_at + o.start + (tid >> 1), (l.act == QMK_ACT_SILU ? t * sigmoid(t) : gelu_tanh(t)) * up);
  } else if (op == OP_IN_PROJECT) {
    const float pair = dpp_f32<kDppQuadXor1>(0.f, t);
    if (mine) {
      const int W = l.mix_width;
      int gate = 0;          // 1: sigmoid, 2: times sigmoid (silu), 3: gelu
      if (!plain && type == QMK_MIXER_RGLRU) {
        t += a[0];
        if (row < W) {
          gate = 3;
        } else {
          if (l.taps > 1) shift_new[static_cast<size_t>(l.taps - 2) * W + row - W] = t;
          t = fmaf(a[2], t, a[1]);
        }
      } else if (!plain && type == QMK_MIXER_LATENT) {
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
      } else if (plain && type == QMK_MIXER_ATTENTION) {
        const int q_rows = l.heads * l.q_stride, k_rows = l.kv_heads * l.head_dim, v_rows = l.kv_heads * l.v_dim;
        const int d = row < q_rows ? row % l.q_stride : row < q_rows + k_rows ? (row - q_rows) % l.head_dim : l.rot_true;
        if (d < l.rot_true) {
          const size_t at = static_cast<size_t>(p.position) * (l.rot_true / 2) + (d >> 1);
          const float c = l.rope_cos[at], sn = l.rope_sin[at];
          t = t * c + ((tid & 1) ? pair * sn : -(pair * sn));
        }
        if (row >= q_rows + k_rows + v_rows) gate = 1;
      } else if (plain && type == QMK_MIXER_DELTA) {
        if (row < channels) {
          if (l.taps > 1) shift_new[static_cast<size_t>(l.taps - 2) * channels + row] = t;
          t = fmaf(a[2], t, a[1]);
          gate = 2;
        } else if (row >= channels + l.rank + l.gate_rank) {
          gate = 1;
        }
      } else if (plain && type == QMK_MIXER_GLA) {
        const int from = 2 * l.heads * l.head_dim + l.heads * l.v_dim;
        if (row >= from && row < from + l.heads * l.v_dim) gate = 2;
      } else if (!plain && row >= 4 * W) {
        t = tanhf(t);
      } else if (!plain && row >= 3 * W) {
        gate = 2;
      }
      if (gate) {
        const float z = gate == 3 ? 1.5957691216057308f * (t + 0.044715f * t * t * t) : t;
        const float sg = sigmoid(z);
        t = gate == 1 ? sg : t * sg;
      }
      st_shared_f32(p.proj + l.proj_at + row, t);
    }
  } else if (!plain && op == OP_LRU_STEP) {
    const float gate = sigmoid(t + a[0]), in_gate = dpp_f32<kDppQuadXor1>(0.f, gate);
    if (mine && !(tid & 1)) {
      const int c = o.start + (tid >> 1);
      const float log_a = gate * a[1];
      const float b = sqrtf(-expm1f(2.f * log_a)) * in_gate * s.xs[xs_at(c)];
      const float now = fmaf(expf(log_a), a[2], b);
      *state = now;
      st_shared_f32(p.mix + o.sub * l.block_dim + c, now * a[3]);
    }
  } else if (!plain && op == OP_LATENT_VALUE) {
    if (mine) st_shared_f32(p.mix + o.sub * l.v_dim + row, t * a[0]);
  } else if (!plain && op == OP_LATENT_ABSORB) {
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
  } else if (!plain && op == OP_WKV_STEP) {
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
  } else if (plain && op == OP_STATE_STEP) {
    // S <- decay S, u = beta (v - S^T k), S <- S + k u^T, o = S^T q, with S^T k and S^T q taken together:
    // o = (decay S)^T q + (q . k) u.  Without the delta rule u = v.
    const bool delta = type == QMK_MIXER_DELTA;
    const int n = o.count, dim = l.head_dim, groups = kThreads / n, e = tid % n, group = tid / n;
    float *q = s.aux, *k = q + kStateVector, *w = k + kStateVector, *v = w + kStateVector;
    if (mine) w[tid] = delta ? delta_decay(l, o.sub, t + a[0]) : gla_decay(l, t + a[0]);
    __syncthreads();
    float ak = 0.f, aq = 0.f;
#pragma unroll
    for (int j0 = 0; j0 < kStateRows; j0 += kStateBatch) {
      if (j0 * groups < dim) {
#pragma unroll
        for (int j = j0; j < j0 + kStateBatch; ++j) {
          const int i = group + j * groups;
          held[j] *= w[i];
          ak = fmaf(k[i], held[j], ak);
          aq = fmaf(q[i], held[j], aq);
        }
      }
    }
    if (group < groups) {
      s.xs[group * n + e] = ak;
      s.xs[(groups + group) * n + e] = aq;
    }
    __syncthreads();
    ak = aq = 0.f;
#pragma unroll 4
    for (int i = 0; i < groups; ++i) {
      ak += s.xs[i * n + e];
      aq += s.xs[(groups + i) * n + e];
    }
    const float u = delta ? a[3] * (v[e] - ak) : v[e];
    if (tid < n) st_shared_f32(p.mix + l.mix_at + o.sub * l.v_dim + o.start + tid, fmaf(a[4], u, aq));
    stamp(p, s, 3);
    arrive_stage(p, o);      // nobody else reads the state in this launch: its stores need no acknowledgement before the arrival
    if (group < groups) {
#pragma unroll
      for (int j0 = 0; j0 < kStateRows; j0 += kStateBatch) {
        if (j0 * groups < dim) {
#pragma unroll
          for (int j = j0; j < j0 + kStateBatch; ++j) {
            const int i = group + j * groups;
            const float now = fmaf(k[i], u, held[j]);
            if (i < dim) state[static_cast<size_t>(i) * l.v_dim] = now;
          }
        }
      }
    }
    return true;
  } else if (plain && op == OP_GATE) {
    if (mine) st_shared_f32(p.proj + l.proj_at + l.in_rows + row, sigmoid(t));
  } else {   // OP_LM_HEAD
    if (plain) t = soft_cap(t * p.logit_scale, p.logit_softcap);
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

// Keys of one tile of OP_ATTEND, and the LDS floats it needs for this cache row width (host and device).
__host__ __device__ constexpr int attend_keys(int element_bytes) { return element_bytes == 2 ? 64 : 32; }
__host__ __device__ constexpr int attend_floats(int row_elements, int element_bytes) {
  const int stride = (row_elements + 31) / 32 * 32 + 8, keys = attend_keys(element_bytes), slices = kWaves / (keys / 16);
  return (16 + keys) * stride * element_bytes / 4 + slices * keys * 16 + keys * 16 + 16 * (keys + 8) + 16;
}

// Part `start` of `count` of the visible keys, sixteen heads.  Scores: matrix tiles of 16 keys x 16 heads, the row's columns
// split over the waves of a tile; then the weights and the running sums of weight x value, of which an instruction keeps
// columns [128 extra, 128 extra + 128), sixteen a wave.
// Latent: heads [16 sub, 16 sub + 16), a row is [latent | rotated key], the latent is the value.  Attention: the heads of key
// head g = sub / b, sixteen of them from 16 (sub % b) on, b = ceil(heads per key head / 16); a row is g's [key | value], and
// the step's own row comes from the projections (one instruction per key head puts it into the cache).
template <class T, bool PLAIN>
__device__ __forceinline__ bool op_attend(const DecodeParams& p, Smem& s, const Op& o) {
  constexpr int kKeys = attend_keys(sizeof(T)), kTiles = kKeys / 16, kSlices = kWaves / kTiles, kPer = kKeys * 16 / kThreads, kSp = kKeys + 8;
  constexpr int kUnit = 16 / sizeof(T);
  LayerRef& l = layer_of(p, o.layer);
  const int heads16 = (l.heads + 15) & ~15;
  constexpr bool latent = !PLAIN;
  if (l.type != (latent ? QMK_MIXER_LATENT : QMK_MIXER_ATTENTION) || o.sub < 0 || o.start < 0 || o.count <= 0 || o.count > p.max_splits || o.start >= o.count || o.extra < 0)
    return bad_operand(p, o, o.start);
  const int group = latent ? l.heads : l.heads / l.kv_heads, blocks = (group + 15) / 16, kv = o.sub / blocks, block = o.sub % blocks;
  const int values = latent ? l.rank : l.v_dim, value_at = latent ? 0 : l.head_dim;      // columns of a row that are its value
  const int head0 = kv * group + block * 16, heads = min(16, group - block * 16);
  if (kv >= (latent ? 1 : l.kv_heads) || o.extra * 16 * kWaves >= values) return bad_operand(p, o, o.sub);
  const int tid = threadIdx.x, lane = tid & (kWaveSize - 1), wave = __builtin_amdgcn_readfirstlane(tid / kWaveSize);
  const int width = latent ? l.rank + l.rot_dim : l.head_dim + l.v_dim, width32 = (width + 31) & ~31, stride = width32 + 8;
  const int pitch = latent ? width : l.kv_heads * width;      // elements between cache rows
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
  T* cache = static_cast<T*>(l.cache) + kv * width;
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
            v[j] = *reinterpret_cast<const v4u*>(cache + static_cast<size_t>(offset + at) * pitch + c * kUnit);
        }
#pragma unroll
        for (int j = 0; j < kBatch; ++j) *reinterpret_cast<v4u*>(sc + (r0 + j * kWaves) * stride + c * kUnit) = v[j];
      }
    }
  };
  // The appended row, where this part holds it (it is then the part's last).
  auto load_appended = [&](int base) {
    if (p.position >= hi || p.position < base || p.position >= base + kKeys) return;
    T* row = cache + static_cast<size_t>(offset + p.position % rows) * pitch;
    if (!latent) {   // neighbouring elements, both of the key or both of the value
      const float* from = p.proj + l.proj_at + l.heads * l.q_stride;
      const bool put = block == 0 && o.extra == 0;
#pragma unroll 1
      for (int c = tid * 2; c < width; c += kThreads * 2) {
        const uint64_t v = ld_shared64(from + (c < l.head_dim ? kv * l.head_dim + c : l.kv_heads * l.head_dim + kv * l.v_dim + c - l.head_dim));
        T* at = sc + (p.position - base) * stride + c;
        at[0] = from_f32<T>(__uint_as_float(static_cast<uint32_t>(v)));
        at[1] = from_f32<T>(__uint_as_float(static_cast<uint32_t>(v >> 32)));
        if (put) {
          row[c] = at[0];
          row[c + 1] = at[1];
        }
      }
      return;
    }
#pragma unroll 1
    for (int c = tid; c * kUnit < width; c += kThreads) *reinterpret_cast<v4u*>(sc + (p.position - base) * stride + c * kUnit) = ld_shared128(row + c * kUnit);
  };
  if (lo < hi) load_tile(lo);
  stamp(p, s, 0);
  if (!wait_stage(p, s, o)) return false;
  if (lo < hi) {
#pragma unroll 1
    for (int k = tid * 2; k < width32; k += kThreads * 2) {
      uint64_t v[16];
      const float* from = !latent ? p.proj + l.proj_at + head0 * l.q_stride + k
                          : k < l.rank ? p.absorbed + head0 * l.rank + k : p.proj + head0 * l.q_stride + l.head_dim + k - l.rank;
      const int step = latent && k < l.rank ? l.rank : l.q_stride, end = latent ? width : l.q_stride;
#pragma unroll
      for (int h = 0; h < 16; ++h) v[h] = h < heads && k < end ? ld_shared64(from + h * step) : 0;
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
  const bool columns = column0 < values;
#pragma unroll 1
  for (int base = lo; base < hi; base += kKeys) {
    if (base != lo) {
      load_tile(base);
      __syncthreads();
      load_appended(base);
    }
    __syncthreads();
    {
      const int tile = wave % kTiles, slice = wave / kTiles, steps = (latent ? width32 : l.q_stride) / 32;
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
        for (int j = 0; j < 8; ++j) cf.set(j, sc[(kk * 32 + (lane >> 4) * 8 + j) * stride + value_at + column0 + (lane & 15)]);
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
  float* ml = p.ml + (static_cast<size_t>(o.start) * heads16 + head0) * 2;
  if (key0 == 0 && o.extra == 0 && (latent || head < heads)) {
    float t = 0.f;
#pragma unroll
    for (int k = 0; k < kWaves; ++k) t += ss[k * 16 + head];
    st_shared_f32(ml + head * 2, m);
    st_shared_f32(ml + head * 2 + 1, t);
  }
  if (columns && (latent || (lane & 15) < heads)) {
    uint64_t* at = reinterpret_cast<uint64_t*>(p.part + (static_cast<size_t>(o.start) * heads16 + head0 + (lane & 15)) * values + column0 + (lane >> 4) * 4);
#pragma unroll
    for (int i = 0; i < 2; ++i)
      __hip_atomic_store(at + i, (static_cast<uint64_t>(__float_as_uint(acc[2 * i + 1])) << 32) | __float_as_uint(acc[2 * i]), __ATOMIC_RELAXED,
                         __HIP_MEMORY_SCOPE_AGENT);
  }
  stamp(p, s, 3);
  arrive_stage(p, o);
  return true;
}

// The parts of one head put together, times its output gate.
__device__ __forceinline__ bool op_attend_merge(const DecodeParams& p, Smem& s, const Op& o) {
  LayerRef& l = layer_of(p, o.layer);
  if (l.type != QMK_MIXER_ATTENTION || o.sub < 0 || o.sub >= l.heads || o.count <= 0 || o.count > p.max_splits || o.count > kMaxParts)
    return bad_operand(p, o, o.sub);
  const int tid = threadIdx.x, heads16 = (l.heads + 15) & ~15, parts = o.count, n = l.v_dim, groups = kThreads / n, e = tid % n, group = tid / n;
  if (!wait_stage(p, s, o)) return false;
  if (tid < parts) {
    const uint64_t ml = ld_shared64(p.ml + (static_cast<size_t>(tid) * heads16 + o.sub) * 2);
    s.aux[tid] = __uint_as_float(static_cast<uint32_t>(ml));
    s.aux[kMaxParts + tid] = __uint_as_float(static_cast<uint32_t>(ml >> 32));
  }
  const float gate = tid < n ? ld_shared_f32(p.proj + l.proj_at + l.heads * l.q_stride + l.kv_heads * (l.head_dim + n) + o.sub * n + tid) : 0.f;
  constexpr int kBatch = 8;
  float v[kBatch];
  const float* column = p.part + static_cast<size_t>(o.sub) * n + e;
  auto request = [&](int base) {
#pragma unroll
    for (int j = 0; j < kBatch; ++j) v[j] = ld_shared_f32(column + static_cast<size_t>(min(base + j * groups, parts - 1)) * heads16 * n);
  };
  request(group);
  __syncthreads();
  if (tid < kWaveSize) {   // weights of the parts
    const float mx = tid < parts ? s.aux[tid] : -INFINITY, top = wave_max(mx);
    const float w = exp2_fast(mx - top), sum = wave_sum(tid < parts ? w * s.aux[kMaxParts + tid] : 0.f);
    s.aux[tid] = tid < parts ? w / sum : 0.f;
  }
  __syncthreads();
  float acc = 0.f;
  if (group < groups) {
#pragma unroll 1
    for (int base = group; base < parts; base += kBatch * groups) {
      if (base != group) request(base);
#pragma unroll
      for (int j = 0; j < kBatch; ++j)
        if (base + j * groups < parts) acc = fmaf(s.aux[base + j * groups], v[j], acc);
    }
    s.xs[group * n + e] = acc;
  }
  __syncthreads();
  if (tid < n) {
    acc = 0.f;
#pragma unroll 4
    for (int i = 0; i < groups; ++i) acc += s.xs[i * n + tid];
    st_shared_f32(p.mix + l.mix_at + o.sub * n + tid, acc * gate);
  }
  arrive_stage(p, o);
  return true;
}

}  // namespace hybrid
}  // namespace qmk
