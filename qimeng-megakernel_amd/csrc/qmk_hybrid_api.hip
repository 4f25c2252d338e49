// The hybrid route's kernels for gfx950 and their C ABI (include/qmk_hybrid.h).
//
// Decode: the persistent interpreter of the other routes (one workgroup per instruction queue, monotone counters with
// bounded waits, the last workgroup to retire clears them) over the ops of qmk_hybrid_ops.h.  Prefill: the launches of
// qmk_hybrid_prefill.h, layer by layer, on the caller's stream.
#include <hip/hip_runtime.h>

#include <algorithm>
#include <mutex>
#include <type_traits>

#include "qmk_hybrid_ops.h"
#include "qmk_hybrid_prefill.h"
#include "qmk_hybrid_plain.h"

namespace qmk {
namespace hybrid {

constexpr int kStatusWords = 8;
constexpr int kMaxDevices = 16;
constexpr int kMaxQueues = 1024;
__device__ int32_t g_status[kStatusWords];

// The launch's parameters as one instruction sees them: read from the kernel-argument segment through a pointer the
// compiler cannot look behind, so that an op loads what it needs of them and keeps nothing across the instruction loop
// (held in scalar registers for the whole kernel they are parked in vector lanes, one move per use).
static_assert(std::is_trivially_copyable<DecodeParams>::value && std::is_standard_layout<DecodeParams>::value, "copied byte for byte into the segment");
__device__ __forceinline__ const DecodeParams& params_of_this_instruction() {
  auto args = __builtin_amdgcn_kernarg_segment_ptr();
  asm volatile("" : "+s"(args));
  return *(const DecodeParams*)args;   // the only kernel argument: offset 0 of the segment
}

template <class T, bool PLAIN>
__global__ __launch_bounds__(kThreads, 1) void decode_megakernel_hybrid(const DecodeParams p_launch) {
  const DecodeParams& p_loop = p_launch;
  __shared__ __align__(16) Smem s;
  if (threadIdx.x == 0) {
    s.best_val = -INFINITY;
    s.best_idx = 0x7fffffff;
  }
  const int num_insts = p_loop.num_insts;
  const int32_t* queue = p_loop.instructions + static_cast<size_t>(blockIdx.x) * num_insts * kInstWords;
  bool ok = true;
  // The words of instruction i + 2 are asked for while instruction i runs.
  int32_t word = (threadIdx.x < kInstWords && num_insts > 0) ? queue[threadIdx.x] : 0;
  int32_t word1 = (threadIdx.x < kInstWords && num_insts > 1) ? queue[kInstWords + threadIdx.x] : 0;
  for (int i = 0; i < num_insts && ok; ++i) {
    if (threadIdx.x < kInstWords) {
      s.inst[threadIdx.x] = word;
      if (threadIdx.x == 1) s.next_layer = word1;
      word = word1;
      word1 = (i + 2 < num_insts) ? queue[(i + 2) * kInstWords + threadIdx.x] : 0;
    }
    __syncthreads();
    const DecodeParams& p = params_of_this_instruction();
    auto operand = [&](int w) { return __builtin_amdgcn_readfirstlane(s.inst[w]); };
    const int next_layer = __builtin_amdgcn_readfirstlane(s.next_layer);
    const Op o{next_layer >= 0 && next_layer < p.num_layers ? next_layer : 0, i, operand(0), operand(1), operand(2), operand(3), operand(4), operand(5), operand(6), operand(7), operand(8)};
    unsigned long long t_start = 0;
    if (p.timeline != nullptr && threadIdx.x == 0) t_start = s.t_wait = wall_clock64();
    if (o.opcode != OP_NOOP && (o.layer < 0 || o.layer >= p.num_layers || o.wait_stage >= 4 * p.groups || o.arrive_stage >= 4 * p.groups)) {
      ok = bad_operand(p, o, o.layer);
    } else {
      switch (o.opcode) {
        case OP_NOOP: break;
        case OP_IN_PROJECT:
        case OP_LRU_STEP:
        case OP_LATENT_ABSORB:
        case OP_LATENT_VALUE:
        case OP_WKV_STEP:
        case OP_OUT_PROJECT:
        case OP_UP_GATE:
        case OP_LM_HEAD:
        case OP_STATE_STEP:
        case OP_JOIN:
        case OP_GATE: ok = op_rows<T, PLAIN>(p, s, o); break;
        case OP_ATTEND: ok = op_attend<T, PLAIN>(p, s, o); break;
        case OP_ATTEND_MERGE:
          if constexpr (PLAIN) ok = op_attend_merge(p, s, o);
          else ok = bad_operand(p, o, o.opcode);
          break;
        default:
          if (threadIdx.x == 0) report_error(counters_of(p), QMK_DEV_BAD_OPCODE, i, o.opcode, 0);
          ok = false;
          break;
      }
    }
    if (p.timeline != nullptr && threadIdx.x == 0) {
      uint64_t* rec = p.timeline + (static_cast<size_t>(blockIdx.x) * p.num_insts + i) * 8;
      rec[0] = t_start;
      rec[1] = s.t_wait;
      rec[2] = wall_clock64();
      rec[3] = static_cast<uint64_t>(o.opcode) | (static_cast<uint64_t>(static_cast<uint32_t>(o.layer)) << 8);
      for (int k = 0; k < 4; ++k) rec[4 + k] = s.stamps[k];
    }
    __syncthreads();
  }
  if (!ok) return;
  const DecodeParams& p = params_of_this_instruction();

  // Retire: the last workgroup to arrive owns the counters alone, clears them and picks the token among the
  // workgroups' candidates (largest logit, smallest row among equals).
  const bool sampling = p.token_out != nullptr;
  if (sampling && threadIdx.x == 0) {
    const uint32_t bits = __float_as_uint(s.best_val);
    const uint32_t key = (bits & 0x80000000u) ? ~bits : (bits | 0x80000000u);
    __hip_atomic_store(p.candidates + blockIdx.x, (static_cast<uint64_t>(key) << 32) | (0xffffffffu - static_cast<uint32_t>(s.best_idx)),
                       __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
  }
  release_stores();
  __syncthreads();
  int32_t* done = counter_ptr(counters_of(p), 0, kStageGroupRows - 1, kStageGroupSlots - 1);
  if (threadIdx.x == 0)
    s.ctl[1] = __hip_atomic_fetch_add(done, 1, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT) == static_cast<int>(gridDim.x) - 1;
  __syncthreads();
  if (!s.ctl[1]) return;
  const int total = p.groups * kStageGroupRows * kStageGroupSlots;
  for (int i = threadIdx.x; i < total; i += kThreads) __hip_atomic_store(p.barriers + i, 0, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
  if (!sampling || threadIdx.x >= kWaveSize) return;
  uint64_t best = 0;
  for (int q = threadIdx.x; q < static_cast<int>(gridDim.x); q += kWaveSize) {
    const uint64_t c = ld_shared64(p.candidates + q);
    best = c > best ? c : best;
  }
  for (int off = 1; off < kWaveSize; off <<= 1) {
    const uint32_t lo = __shfl_xor(static_cast<uint32_t>(best), off), hi = __shfl_xor(static_cast<uint32_t>(best >> 32), off);
    const uint64_t other = (static_cast<uint64_t>(hi) << 32) | lo;
    best = other > best ? other : best;
  }
  const uint32_t token = 0xffffffffu - static_cast<uint32_t>(best);
  if (threadIdx.x == 0 && token < static_cast<uint32_t>(p.vocab)) *p.token_out = token;
}

struct DeviceInfo {
  bool ready = false;
  int max_queues = 0;
  int32_t* status = nullptr;
};
DeviceInfo g_devices[kMaxDevices];
std::mutex g_mutex;

int device_info(DeviceInfo** out) {
  int dev = -1;
  if (hipGetDevice(&dev) != hipSuccess || dev < 0 || dev >= kMaxDevices) return QMK_ERR_NO_DEVICE;
  std::lock_guard<std::mutex> lock(g_mutex);
  DeviceInfo& d = g_devices[dev];
  if (!d.ready) {
    hipDeviceProp_t prop;
    int blocks = kMaxQueues;
    auto fits = [&](auto kernel) {
      int n = 0;
      if (hipOccupancyMaxActiveBlocksPerMultiprocessor(&n, kernel, kThreads, 0) != hipSuccess) return false;
      blocks = std::min(blocks, n);
      return true;
    };
    void* sym = nullptr;
    if (hipGetDeviceProperties(&prop, dev) != hipSuccess || !fits(decode_megakernel_hybrid<u16, false>) || !fits(decode_megakernel_hybrid<float, false>) ||
        !fits(decode_megakernel_hybrid<u16, true>) || !fits(decode_megakernel_hybrid<float, true>) || hipGetSymbolAddress(&sym, HIP_SYMBOL(g_status)) != hipSuccess || hipMemset(sym, 0, sizeof(int32_t) * kStatusWords) != hipSuccess)
      return QMK_ERR_NO_DEVICE;
    d.max_queues = std::min(blocks * prop.multiProcessorCount, kMaxQueues);
    d.status = static_cast<int32_t*>(sym);
    d.ready = true;
  }
  *out = &d;
  return QMK_OK;
}

inline size_t align_up(size_t n) { return (n + 255) & ~size_t(255); }
inline bool m16(int v) { return v > 0 && v % 16 == 0; }
inline int element(const QmkHybridArgs* a) { return a->dtype == QMK_HYBRID_F32 ? 4 : 2; }

// Entries of a plain residual: where they read x, and how a run's branches stand in the table.
bool plain_ok(const QmkHybridArgs* a, int i) {
  const QmkHybridLayer& l = a->layers[i];
  const bool run = l.type >= QMK_MIXER_GLA && l.type <= QMK_MIXER_DELTA;
  if (!run && l.type != QMK_ENTRY_JOIN && l.type != QMK_ENTRY_FINAL) return false;
  if ((i + 1 == a->num_layers) != (l.type == QMK_ENTRY_FINAL)) return false;
  if (l.branch < 0 || l.branches < 1 || l.branches > QMK_HYBRID_MAX_BRANCHES || l.branch >= l.branches || (!run && l.branches != 1)) return false;
  if (i - l.branch < 0 || i - l.branch + l.branches > a->num_layers) return false;
  for (int b = 0; b < l.branches; ++b) {
    const QmkHybridLayer& other = a->layers[i - l.branch + b];
    if (other.branch != b || other.branches != l.branches || (b > 0 && other.has_mlp)) return false;
  }
  if (l.x_from < -1 || l.x_from > 1 || l.x_to < 0 || l.x_to > 1 || l.x_from == l.x_to) return false;
  if (l.prev < -1 || l.prev >= i || (l.prev >= 0 && (a->layers[l.prev].branch != 0 || a->layers[l.prev].type > QMK_MIXER_DELTA || l.x_from < 0))) return false;
  return l.norm >= QMK_NORM_RMS && l.norm <= QMK_NORM_LAYER && l.proj_at >= 0 && l.proj_at % 16 == 0 && l.mix_at >= 0 && l.mix_at % 16 == 0 && l.ff_at >= 0 &&
         l.ff_at % 16 == 0;
}

bool layer_ok(const QmkHybridArgs* a, int i) {
  const QmkHybridLayer& l = a->layers[i];
  if (a->streams == 0 ? !plain_ok(a, i) : l.type > QMK_MIXER_WKV) return false;
  if (l.type == QMK_ENTRY_JOIN) return 2 * a->width <= kMaxK;
  if (l.type == QMK_ENTRY_FINAL) return true;
  if (!m16(l.in_rows) || !m16(l.mix_width) || l.mix_width > kMaxK) return false;
  if (l.has_mlp && (!m16(l.ff) || l.ff > kMaxK)) return false;
  switch (l.type) {
    case QMK_MIXER_RGLRU:
      return l.taps >= 1 && l.taps <= kMaxTaps && l.blocks > 0 && m16(l.block_dim) && l.blocks * l.block_dim == l.mix_width && l.in_rows == 2 * l.mix_width;
    case QMK_MIXER_LATENT:
      return l.heads > 0 && m16(l.head_dim) && m16(l.rot_dim) && l.rot_true > 0 && l.rot_true % 2 == 0 && l.rot_true <= l.rot_dim && m16(l.v_dim) &&
             l.v_dim <= 256 && m16(l.rank) && l.rank <= kMaxRank && l.rank_true > 0 && l.rank_true <= l.rank && l.q_stride % 32 == 0 &&
             l.q_stride >= l.head_dim + l.rot_dim && l.q_stride <= 256 && l.window > 0 && l.ring > 0 && l.mix_width == l.heads * l.v_dim &&
             l.in_rows == l.heads * (l.q_stride + l.v_dim) + l.rank + l.rot_dim &&
             attend_floats(l.rank + l.rot_dim, element(a)) <= kAttendFloats;
    case QMK_MIXER_WKV:
      return l.heads > 0 && m16(l.head_dim) && l.head_dim <= kMaxHeadDim && l.head_dim_true > 0 && l.head_dim_true <= l.head_dim && m16(l.rank) &&
             l.rank <= kMaxK && l.mix_width == l.heads * l.head_dim && l.in_rows == 4 * l.mix_width + l.rank;
    case QMK_MIXER_ATTENTION:
      return l.heads > 0 && l.kv_heads > 0 && l.heads % l.kv_heads == 0 && m16(l.head_dim) && m16(l.v_dim) && l.v_dim <= 256 && l.rot_dim == 0 &&
             l.rot_true >= 0 && l.rot_true % 2 == 0 && l.rot_true <= l.head_dim && l.q_stride == (l.head_dim + 31) / 32 * 32 && l.q_stride <= 256 &&
             l.window > 0 && l.ring > 0 && l.mix_width == l.heads * l.v_dim &&
             l.in_rows == l.heads * (l.q_stride + l.v_dim) + l.kv_heads * (l.head_dim + l.v_dim) &&
             attend_floats(l.head_dim + l.v_dim, element(a)) <= kAttendFloats;
    case QMK_MIXER_GLA:
    case QMK_MIXER_DELTA: {
      const bool delta = l.type == QMK_MIXER_DELTA;
      if (l.heads < 1 || l.kv_heads < 1 || l.heads % l.kv_heads != 0 || !m16(l.head_dim) || l.head_dim > kMaxHeadDim || !m16(l.v_dim) || l.v_dim > kMaxHeadDim ||
          l.v_true < 1 || l.v_true > l.v_dim || !m16(l.rank) || l.mix_width != l.heads * l.v_dim)
        return false;
      if (!delta) return l.kv_heads == l.heads && l.gate_rank == 0 && l.rank <= kMaxK && l.in_rows == 2 * l.heads * (l.head_dim + l.v_dim) + l.rank;
      return m16(l.gate_rank) && l.rank + l.gate_rank <= kMaxK && l.taps >= 1 && l.taps <= kMaxTaps &&
             l.in_rows == conv_channels(l) + l.rank + l.gate_rank + (l.heads + 15) / 16 * 16;
    }
    default: return false;
  }
}

int check_shape(const QmkHybridArgs* a) {
  if (a == nullptr || a->layers == nullptr) return QMK_ERR_NULL_ARG;
  if (a->struct_size != sizeof(QmkHybridArgs)) return QMK_ERR_ABI;
  if (a->dtype > QMK_HYBRID_F32) return QMK_ERR_MODEL;
  if (a->num_layers < 1 || !m16(a->width) || a->width > kMaxK || a->width_true < 1 || a->width_true > a->width || a->streams < 0 ||
      a->streams > kMaxStreams || a->vocab < 1 || !m16(a->vocab_rows) || a->vocab > a->vocab_rows || !(a->eps >= 0.f) ||
      !(a->logit_softcap >= 0.f))
    return QMK_ERR_SHAPE;
  for (int i = 0; i < a->num_layers; ++i)
    if (!layer_ok(a, i)) return QMK_ERR_SHAPE;
  return QMK_OK;
}

bool layer_pointers(const QmkHybridLayer& l) {
  if (l.type == QMK_ENTRY_JOIN) return l.in_w != nullptr;
  if (l.type == QMK_ENTRY_FINAL) return l.norm1 != nullptr;
  if (l.type >= QMK_MIXER_GLA) {
    bool ok = l.in_w && l.o_w && (l.branch > 0 || l.norm1) && (!l.has_mlp || (l.mlp_w && l.down_w)) && (l.branches > 1) == (l.out_norm != nullptr);
    if (l.type == QMK_MIXER_ATTENTION) return ok && l.cache && ((l.rope_cos && l.rope_sin) || l.rot_true == 0);
    ok = ok && l.mid_w && l.mid_b && l.vec0 && l.state;
    return ok && (l.type == QMK_MIXER_GLA || (l.gate_w && l.vec1 && l.vec2 && (l.shift || l.taps == 1)));
  }
  bool ok = l.norm1 && l.in_w && l.mid_w && l.vec0;
  if (l.type == QMK_MIXER_LATENT) ok = ok && l.uk_w && l.uv_w && l.rope_cos && l.rope_sin && l.cache;
  else ok = ok && l.mid_b && l.vec1 && l.vec2 && l.state && (l.shift || (l.type == QMK_MIXER_RGLRU && l.taps == 1));
  if (l.type == QMK_MIXER_RGLRU) ok = ok && l.in_b;
  if (l.has_mlp) ok = ok && l.norm2 && l.mlp_w && l.down_w && l.next2;
  return ok && l.o_w && l.hc && l.next1;
}

int check_launch(const QmkHybridArgs* a, int tokens) {
  if (int rc = check_shape(a); rc != QMK_OK) return rc;
  if (!a->layers_device || !a->embed || !a->final_norm || !a->head || !a->token_in || !a->workspace) return QMK_ERR_NULL_ARG;
  for (int i = 0; i < a->num_layers; ++i)
    if (!layer_pointers(a->layers[i])) return QMK_ERR_NULL_ARG;
  if (a->slots < 1 || a->slot < 0 || a->slot >= a->slots || (a->flip != 0 && a->flip != 1)) return QMK_ERR_SHAPE;
  if (tokens < 1 || a->position < 0 || a->position > a->max_positions - tokens) return QMK_ERR_POSITION;
  for (int i = 0; i < a->num_layers; ++i) {
    const QmkHybridLayer& l = a->layers[i];
    // every key a query of the launch sees must still have its row when the launch's rows have been written
    if ((l.type == QMK_MIXER_LATENT || l.type == QMK_MIXER_ATTENTION) && l.ring < std::min(a->position + tokens, l.window - 1 + tokens)) return QMK_ERR_SHAPE;
  }
  if (reinterpret_cast<uintptr_t>(a->workspace) % 256 != 0) return QMK_ERR_SHAPE;
  return QMK_OK;
}

struct Carver {
  char* base;
  size_t used = 0;
  template <class T>
  T* take(size_t n) {
    T* t = base == nullptr ? nullptr : reinterpret_cast<T*>(base + used);
    used += align_up(n * sizeof(T));
    return t;
  }
};

struct DecodeBuffers {
  uint64_t* candidates;
  float *u, *x, *out, *proj, *mix, *absorbed, *part, *ml;
};
size_t decode_buffers(const QmkHybridArgs* a, void* base, DecodeBuffers* b) {
  size_t proj = 0, mix = 0, absorbed = 0, part = 0, ml = 0;
  for (int i = 0; i < a->num_layers; ++i) {
    const QmkHybridLayer& l = a->layers[i];
    if (l.type > QMK_MIXER_DELTA) continue;
    proj = std::max<size_t>(proj, static_cast<size_t>(l.proj_at) + l.in_rows + (l.type == QMK_MIXER_DELTA ? l.mix_width : 0));
    mix = std::max<size_t>(mix, std::max(static_cast<size_t>(l.mix_at) + l.mix_width, l.has_mlp ? static_cast<size_t>(l.ff_at) + l.ff : 0));
    if (l.type == QMK_MIXER_ATTENTION) {
      const size_t heads16 = (l.heads + 15) & ~15;
      part = std::max(part, a->max_splits * heads16 * l.v_dim);
      ml = std::max(ml, a->max_splits * heads16 * 2);
    }
    if (l.type == QMK_MIXER_LATENT) {
      const size_t heads16 = (l.heads + 15) & ~15;
      absorbed = std::max<size_t>(absorbed, static_cast<size_t>(l.heads) * l.rank);
      part = std::max(part, a->max_splits * heads16 * l.rank);
      ml = std::max(ml, a->max_splits * heads16 * 2);
    }
  }
  Carver c{static_cast<char*>(base)};
  b->candidates = c.take<uint64_t>(kMaxQueues);
  b->u = c.take<float>(a->width);
  b->x = c.take<float>(static_cast<size_t>(a->streams > 0 ? a->streams : 2) * a->width);
  b->out = c.take<float>(a->streams > 0 ? 0 : static_cast<size_t>(QMK_HYBRID_MAX_BRANCHES + 1) * a->width);
  b->proj = c.take<float>(proj);
  b->mix = c.take<float>(mix);
  b->absorbed = c.take<float>(absorbed);
  b->part = c.take<float>(part);
  b->ml = c.take<float>(ml);
  return c.used;
}

inline size_t values_cap(const QmkHybridArgs* a) { return (static_cast<size_t>(a->max_positions) + 31) & ~size_t(31); }

template <class T>
struct PlainBuffers {
  float *x, *branch, *qkv, *values, *decay, *beta, *o, *chunks;
  T *h, *q, *low, *gate, *mix, *vt;
};
template <class T>
size_t plain_buffers(const QmkHybridArgs* a, void* base, PlainBuffers<T>* b) {
  const size_t P = a->portion_rows, D = a->width, chunks_of = (P + kChunkTokens - 1) / kChunkTokens;
  size_t h = P * D, branch = 0, qkv = 0, values = 0, decay = 0, beta = 0, o = 0, chunks = 0, q = 0, low = 0, gate = 0, mix = 0, vt = 0;
  for (int i = 0; i < a->num_layers; ++i) {
    const QmkHybridLayer& l = a->layers[i];
    if (l.type == QMK_ENTRY_JOIN) h = std::max(h, 2 * P * D);
    if (l.type > QMK_MIXER_DELTA) continue;
    mix = std::max(mix, P * std::max<size_t>(l.mix_width, l.has_mlp ? l.ff : 0));
    gate = std::max(gate, P * l.mix_width);
    if (l.branches > 1) branch = std::max(branch, l.branches * P * D);
    if (l.type == QMK_MIXER_ATTENTION) {
      q = std::max(q, P * l.heads * l.q_stride);
      vt = std::max(vt, values_cap(a) * l.kv_heads * l.v_dim);
      continue;
    }
    decay = std::max(decay, P * l.heads * l.head_dim);
    o = std::max(o, P * l.mix_width);
    low = std::max(low, P * (l.rank + l.gate_rank));
    chunks = std::max(chunks, chunks_of * l.heads * chunk_floats(l.head_dim));
    if (l.type == QMK_MIXER_DELTA) {
      qkv = std::max(qkv, P * conv_channels(l));
      values = std::max(values, P * l.mix_width);
      beta = std::max(beta, P * ((l.heads + 15) / 16 * 16));
    } else {
      qkv = std::max(qkv, P * (2 * l.heads * l.head_dim + l.mix_width));
    }
  }
  Carver c{static_cast<char*>(base)};
  PlainBuffers<T> local;
  if (b == nullptr) b = &local;
  b->x = c.take<float>(P * D);
  b->branch = c.take<float>(branch);
  b->qkv = c.take<float>(qkv);
  b->values = c.take<float>(values);
  b->decay = c.take<float>(decay);
  b->beta = c.take<float>(beta);
  b->o = c.take<float>(o);
  b->chunks = c.take<float>(chunks);
  b->h = c.take<T>(h);
  b->q = c.take<T>(q);
  b->low = c.take<T>(low);
  b->gate = c.take<T>(gate);
  b->mix = c.take<T>(mix);
  b->vt = c.take<T>(vt);
  return c.used;
}

inline int keys_cap(const QmkHybridArgs* a, const QmkHybridLayer& l) { return (std::min(l.window - 1 + a->portion_rows, a->max_positions) + 31) & ~31; }

template <class T>
struct PrefillBuffers {
  float *x, *u, *fa, *fb, *raw;
  T *h, *p0, *p1, *p2, *mix, *rows, *kn, *vt;
};
template <class T>
size_t prefill_buffers(const QmkHybridArgs* a, void* base, PrefillBuffers<T>* b) {
  if (a->streams == 0) return plain_buffers<T>(a, base, nullptr);
  const size_t P = a->portion_rows, D = a->width;
  size_t h = P * D, fa = 0, fb = 0, raw = 0, p0 = 0, p1 = 0, p2 = 0, mix = 0, rows = 0, kn = 0, vt = 0;
  for (int i = 0; i < a->num_layers; ++i) {
    const QmkHybridLayer& l = a->layers[i];
    const size_t W = l.mix_width;
    mix = std::max(mix, P * std::max<size_t>(W, l.has_mlp ? l.ff : 0));
    if (l.type == QMK_MIXER_RGLRU) {
      p0 = std::max(p0, P * W);
      p1 = std::max(p1, P * W);
      p2 = std::max(p2, P * W);
      fa = std::max(fa, P * W);
      fb = std::max(fb, P * W);
    } else if (l.type == QMK_MIXER_LATENT) {
      const size_t keys = keys_cap(a, l);
      p0 = std::max(p0, P * l.heads * l.q_stride);
      p1 = std::max(p1, P * W);
      raw = std::max(raw, P * (l.rank + l.rot_dim));
      rows = std::max(rows, keys * (l.rank + l.rot_dim));
      kn = std::max(kn, keys * l.heads * l.head_dim);
      vt = std::max(vt, keys * W);
    } else {
      h = std::max(h, 5 * P * D);
      p0 = std::max(p0, P * W);
      p1 = std::max(p1, P * l.rank);
      fa = std::max(fa, 3 * P * W);
      fb = std::max(fb, P * W);
      raw = std::max(raw, P * W);
    }
  }
  Carver c{static_cast<char*>(base)};
  b->x = c.take<float>(P * a->streams * D);
  b->u = c.take<float>(P * D);
  b->fa = c.take<float>(fa);
  b->fb = c.take<float>(fb);
  b->raw = c.take<float>(raw);
  b->h = c.take<T>(h);
  b->p0 = c.take<T>(p0);
  b->p1 = c.take<T>(p1);
  b->p2 = c.take<T>(p2);
  b->mix = c.take<T>(mix);
  b->rows = c.take<T>(rows);
  b->kn = c.take<T>(kn);
  b->vt = c.take<T>(vt);
  return c.used;
}

// Large tiles where they fill the chip, small ones otherwise.
template <class TA, class TW, class T>
void launch_gemm(const GemmArgs& g, hipStream_t st) {
  const int n = std::max(g.N, g.last_n);
  auto grid = [&](int bm, int bn) { return dim3((n + bn - 1) / bn, (g.M + bm - 1) / bm, g.groups); };
  const dim3 large = grid(128, 128), block(kPfThreads);
  const bool fills = static_cast<long long>(large.x) * large.y * large.z >= 192;
  if constexpr (sizeof(TA) == 2 && sizeof(TW) == 2) {
    if (g.K % 64 == 0) {
      if (fills) hipLaunchKernelGGL((gemm_direct<T, 128, 128, 2>), large, block, 0, st, g);
      else hipLaunchKernelGGL((gemm_direct<T, 64, 64, 4>), grid(64, 64), block, 0, st, g);
      return;
    }
  }
  if (fills) hipLaunchKernelGGL((gemm<TA, TW, T, 128, 128>), large, block, 0, st, g);
  else hipLaunchKernelGGL((gemm<TA, TW, T, 64, 64>), grid(64, 64), block, 0, st, g);
}

// rows: where the rotated part of a latent attention's keys is, behind the latent.
template <class T>
void launch_attention(const QmkHybridArgs* a, const QmkHybridLayer& l, const T* q, Keys<T> keys, const T* rows, const T* vt, const T* gate, int first, int cap, T* out,
                      hipStream_t st) {
  auto launch = [&](auto kernel) {
    hipLaunchKernelGGL(kernel, dim3((a->tokens + 63) / 64, l.heads), dim3(kPfThreads), 0, st, q, keys, rows, vt, gate, l, first, a->position, a->tokens, cap, out);
  };
  if (l.q_stride <= 128 && l.v_dim <= 64) launch(window_attention<T, 4, 4>);
  else if (l.q_stride <= 128 && l.v_dim <= 128) launch(window_attention<T, 4, 8>);
  else if (l.q_stride <= 192 && l.v_dim <= 128) launch(window_attention<T, 6, 8>);
  else launch(window_attention<T, 8, 16>);
}

template <class T>
int prefill_plain(const QmkHybridArgs* a);

template <class T>
int prefill(const QmkHybridArgs* a) {
  if (a->streams == 0) return prefill_plain<T>(a);
  PrefillBuffers<T> b;
  if (prefill_buffers<T>(a, a->workspace, &b) > a->workspace_bytes) return QMK_ERR_SCRATCH;
  const hipStream_t st = static_cast<hipStream_t>(a->stream);
  const int M = a->tokens, D = a->width, S = a->streams, P = a->portion_rows;
  const dim3 block(kPfThreads);
  hipLaunchKernelGGL(embed_tokens, dim3(M), block, 0, st, a->embed, a->token_in, a->vocab, a->layers[0].hc, S, D, b.x, b.u);
  auto gemm_args = [&](const T* in, int lda, const u16* w, int N, int K, const QmkHybridLayer& l, int epi) {
    GemmArgs g{};
    g.a = in; g.lda = lda; g.w = w; g.ldw = K; g.M = M; g.N = g.last_n = N; g.K = K; g.groups = 1;
    g.layer = l; g.epi = epi; g.position = a->position; g.streams = S; g.width = D; g.rows_cap = P;
    return g;
  };
  auto residual = [&](const u16* w, int K, const QmkHybridLayer& l, bool down) {
    GemmArgs g = gemm_args(b.mix, K, w, D, K, l, EPI_RESIDUAL);
    g.f0 = b.x; g.f1 = b.u; g.down = down; g.next = down ? l.next2 : l.next1;
    launch_gemm<T, u16, T>(g, st);
  };
  for (int i = 0; i < a->num_layers; ++i) {
    const QmkHybridLayer& l = a->layers[i];
    const int W = l.mix_width;
    if (l.type != QMK_MIXER_WKV)
      hipLaunchKernelGGL(norm_rows<T>, dim3(M), block, 0, st, b.u, l.norm1, nullptr, M, D, a->width_true, a->eps, b.h);
    if (l.type == QMK_MIXER_RGLRU) {
      GemmArgs g = gemm_args(b.h, D, l.in_w, l.in_rows, D, l, EPI_RGLRU_IN);
      g.out = b.p0; g.out2 = b.p1;
      launch_gemm<T, u16, T>(g, st);
      const long long quads = static_cast<long long>(M) * (W / 4);
      hipLaunchKernelGGL(causal_conv<T>, dim3(static_cast<unsigned>((quads + kPfThreads - 1) / kPfThreads)), block, 0, st, b.p1, l, a->slot, a->flip, M, b.p2);
      GemmArgs e = gemm_args(b.p2, W, l.mid_w, 2 * l.block_dim, l.block_dim, l, EPI_LRU_GATES);
      e.groups = l.blocks; e.a_step = l.block_dim; e.w_step = 2LL * l.block_dim * l.block_dim;
      e.src = b.p2; e.f0 = b.fa; e.f1 = b.fb;
      launch_gemm<T, u16, T>(e, st);
      hipLaunchKernelGGL(lru_scan<T>, dim3(W / kScanChannels), dim3(kScanChannels * kScanRuns), 0, st, b.fa, b.fb, b.p0, l, a->slot, M, b.mix);
    } else if (l.type == QMK_MIXER_LATENT) {
      GemmArgs g = gemm_args(b.h, D, l.in_w, l.in_rows, D, l, EPI_LATENT_IN);
      g.out = b.p0; g.out2 = b.p1; g.f0 = b.raw;
      launch_gemm<T, u16, T>(g, st);
      const int first = std::max(0, a->position + 1 - l.window), keys = a->position + M - first, cap = keys_cap(a, l), width = l.rank + l.rot_dim;
      hipLaunchKernelGGL(latent_rows<T>, dim3(keys), block, 0, st, b.raw, l, a->slot, first, a->position, a->eps, b.rows);
      GemmArgs k = gemm_args(b.rows, width, l.uk_w, l.heads * l.head_dim, l.rank, l, EPI_STORE);
      k.M = keys; k.out = b.kn; k.ldo = l.heads * l.head_dim;
      launch_gemm<T, u16, T>(k, st);
      GemmArgs v = gemm_args(nullptr, l.rank, nullptr, keys, l.rank, l, EPI_STORE);   // transposed: W_uv rows x keys
      v.a = l.uv_w; v.w = b.rows; v.ldw = width; v.M = l.heads * l.v_dim; v.out = b.vt; v.ldo = cap;
      launch_gemm<u16, T, T>(v, st);
      const Keys<T> expanded{b.kn, l.heads * l.head_dim, l.head_dim, 1};
      launch_attention<T>(a, l, b.p0, expanded, b.rows, b.vt, b.p1, first, cap, b.mix, st);
    } else {
      const int N = W, n = l.head_dim;
      hipLaunchKernelGGL(shift_mix<T>, dim3(M), block, 0, st, b.u, l, a->slot, a->flip, M, P, D, a->width_true, a->eps, b.h);
      GemmArgs g = gemm_args(b.h, D, l.in_w, N, D, l, EPI_WKV_IN);
      g.groups = 5; g.last_n = l.rank; g.a_step = static_cast<long long>(P) * D; g.w_step = static_cast<long long>(N) * D;
      g.f0 = b.fa; g.out = b.p0; g.out2 = b.p1;
      launch_gemm<T, u16, T>(g, st);
      GemmArgs d = gemm_args(b.p1, l.rank, l.mid_w, N, l.rank, l, EPI_WKV_DECAY);
      d.f0 = b.fb; d.ldo = N;
      launch_gemm<T, u16, T>(d, st);
      const size_t step = static_cast<size_t>(P) * N;
      const dim3 grid(n / kWkvColumns, l.heads), lanes(kWkvThreads);
      const float *r = b.fa, *k = b.fa + step, *v = b.fa + 2 * step;
      if (n <= 64) hipLaunchKernelGGL((wkv_scan<4, 32>), grid, lanes, 0, st, r, k, v, b.fb, l, a->slot, M, b.raw);
      else if (n <= 128) hipLaunchKernelGGL((wkv_scan<8, 16>), grid, lanes, 0, st, r, k, v, b.fb, l, a->slot, M, b.raw);
      else hipLaunchKernelGGL((wkv_scan<16, 8>), grid, lanes, 0, st, r, k, v, b.fb, l, a->slot, M, b.raw);
      hipLaunchKernelGGL(wkv_out<T>, dim3((M * l.heads + 3) / 4), block, 0, st, b.raw, b.p0, l, M, a->eps, b.mix);
    }
    residual(l.o_w, W, l, false);
    if (l.has_mlp) {
      hipLaunchKernelGGL(norm_rows<T>, dim3(M), block, 0, st, b.u, l.norm2, nullptr, M, D, a->width_true, a->eps, b.h);
      GemmArgs g = gemm_args(b.h, D, l.mlp_w, 2 * l.ff, D, l, EPI_GEGLU);
      g.out = b.mix;
      launch_gemm<T, u16, T>(g, st);
      residual(l.down_w, l.ff, l, true);
    }
    if (a->layer_out != nullptr)
      hipLaunchKernelGGL(sum_streams, dim3(M), block, 0, st, b.x, S, D, a->layer_out + static_cast<size_t>(i) * M * D);
  }
  if (a->num_want > 0) {
    hipLaunchKernelGGL(norm_rows<T>, dim3(a->num_want), block, 0, st, b.u, a->final_norm, a->want, M, D, a->width_true, a->eps, b.h);
    GemmArgs g = gemm_args(b.h, D, a->head, a->vocab_rows, D, a->layers[0], EPI_LOGITS);
    g.M = a->num_want; g.f0 = a->logits; g.ldo = a->vocab_rows;
    launch_gemm<T, u16, T>(g, st);
  }
  return hipGetLastError() == hipSuccess ? QMK_OK : QMK_ERR_LAUNCH;
}

// The recurrence of a gla or delta entry over the portion, from its projections to what its output projection reads.
template <bool DELTA>
void run_chunks(const QmkHybridArgs* a, const ChunkArgs& g, hipStream_t st) {
  const QmkHybridLayer& l = g.layer;
  const int chunks = (g.M + kChunkTokens - 1) / kChunkTokens, tiles = wave_tiles(l.head_dim);
  hipLaunchKernelGGL(chunk_prepare<DELTA>, dim3(chunks, l.heads), dim3(kPfThreads), 0, st, g);
  const dim3 grid(l.heads, l.v_dim / 16), block(kChunkWaves * 64);
  if (tiles == 1) hipLaunchKernelGGL((chunk_scan<1, DELTA>), grid, block, 0, st, g);
  else if (tiles == 2) hipLaunchKernelGGL((chunk_scan<2, DELTA>), grid, block, 0, st, g);
  else hipLaunchKernelGGL((chunk_scan<4, DELTA>), grid, block, 0, st, g);
}

template <class T>
int prefill_plain(const QmkHybridArgs* a) {
  PlainBuffers<T> b;
  if (plain_buffers<T>(a, a->workspace, &b) > a->workspace_bytes) return QMK_ERR_SCRATCH;
  const hipStream_t st = static_cast<hipStream_t>(a->stream);
  const int M = a->tokens, D = a->width;
  const size_t rows = static_cast<size_t>(a->portion_rows) * D;
  const dim3 block(kPfThreads);
  auto gemm_args = [&](const T* in, const u16* w, int N, int K, const QmkHybridLayer& l, int epi) {
    GemmArgs g{};
    g.a = in; g.lda = K; g.w = w; g.ldw = K; g.M = M; g.N = g.last_n = N; g.K = K; g.groups = 1;
    g.layer = l; g.epi = epi; g.position = a->position; g.slot = a->slot; g.width = D; g.ldo = D;
    g.logit_scale = a->logit_scale; g.logit_softcap = a->logit_softcap;
    return g;
  };
  int runs_done = 0;
  // x as entry l reads it: its norm (or [x; embedding]) -> h; `want`: of those rows alone, x stays.
  auto residual = [&](const QmkHybridLayer& l, const int32_t* want, int count, bool added, float* dump) {
    ResidualArgs g{};
    g.x = b.x; g.table = a->embed; g.tokens = a->token_in; g.vocab = a->vocab; g.want = want; g.dump = dump;
    g.weight = l.type == QMK_ENTRY_JOIN ? nullptr : l.norm1;
    g.embed = l.x_from < 0; g.M = M; g.D = D; g.width = a->width_true; g.norm = l.norm; g.eps = a->eps;
    if (added && l.prev >= 0 && a->layers[l.prev].branches == 2) {
      const QmkHybridLayer* before = a->layers + l.prev;
      g.a = b.branch; g.b = b.branch + rows; g.wa = before[0].out_norm; g.wb = before[1].out_norm; g.scale = before[0].out_scale;
    }
    hipLaunchKernelGGL(residual_rows<T>, dim3(count), block, 0, st, g, b.h);
  };
  auto dump_of = [&](const QmkHybridLayer& l) {   // where the run before this entry is asked for
    return a->layer_out != nullptr && l.prev >= 0 ? a->layer_out + static_cast<size_t>(runs_done++) * M * D : nullptr;
  };
  for (int i = 0; i < a->num_layers; ++i) {
    const QmkHybridLayer& l = a->layers[i];
    const int W = l.mix_width;
    if (l.type == QMK_ENTRY_FINAL) {
      float* dump = dump_of(l);
      if (dump != nullptr) residual(l, nullptr, M, true, dump);     // (and x is complete)
      if (a->num_want > 0) {
        residual(l, a->want, a->num_want, dump == nullptr, nullptr);
        GemmArgs g = gemm_args(b.h, a->head, a->vocab_rows, D, l, EPI_CAPPED_LOGITS);
        g.M = a->num_want; g.f0 = a->logits; g.ldo = a->vocab_rows;
        launch_gemm<T, u16, T>(g, st);
      }
      break;
    }
    if (l.branch == 0) residual(l, nullptr, M, true, dump_of(l));
    if (l.type == QMK_ENTRY_JOIN) {
      GemmArgs g = gemm_args(b.h, l.in_w, D, 2 * D, l, EPI_LOGITS);
      g.f0 = b.x;
      launch_gemm<T, u16, T>(g, st);
      continue;
    }
    if (l.type == QMK_MIXER_ATTENTION) {
      GemmArgs g = gemm_args(b.h, l.in_w, l.in_rows, D, l, EPI_ATTENTION_IN);
      g.out = b.q; g.out2 = b.gate;
      launch_gemm<T, u16, T>(g, st);
      const int row = l.head_dim + l.v_dim, pitch = l.kv_heads * row, keys = a->position + M, cap = static_cast<int>(values_cap(a));
      const T* cache = static_cast<const T*>(l.cache) + static_cast<size_t>(a->slot) * l.ring * pitch;
      hipLaunchKernelGGL(transpose_values<T>, dim3((keys + 63) / 64, (l.v_dim + 63) / 64, l.kv_heads), block, 0, st, cache, pitch, row, l.head_dim, l.v_dim, keys, cap, b.vt);
      launch_attention<T>(a, l, b.q, Keys<T>{cache, pitch, row, l.heads / l.kv_heads}, nullptr, b.vt, b.gate, 0, cap, b.mix, st);
    } else {
      ChunkArgs c{};
      c.layer = l; c.decay = b.decay; c.chunks = b.chunks; c.out = b.o; c.M = M; c.slot = a->slot; c.flip = a->flip;
      if (l.type == QMK_MIXER_DELTA) {
        const int channels = conv_channels(l), ranks = l.rank + l.gate_rank, beta_ld = (l.heads + 15) / 16 * 16;
        GemmArgs g = gemm_args(b.h, l.in_w, l.in_rows, D, l, EPI_DELTA_IN);
        g.f1 = b.qkv; g.out2 = b.low; g.f0 = b.beta; g.ldo = beta_ld;
        launch_gemm<T, u16, T>(g, st);
        const int keys = l.heads * l.head_dim;
        GemmArgs e = gemm_args(b.low, l.mid_w, keys, l.rank, l, EPI_DELTA_DECAY);
        e.lda = ranks; e.f0 = b.decay; e.ldo = keys;
        launch_gemm<T, u16, T>(e, st);
        GemmArgs f = gemm_args(b.low + l.rank, l.gate_w, W, l.gate_rank, l, EPI_SIGMOID);
        f.lda = ranks; f.out = b.gate; f.ldo = W;
        launch_gemm<T, u16, T>(f, st);
        c.qkv = b.qkv; c.beta = b.beta; c.beta_ld = beta_ld; c.values = b.values; c.value_ld = W;
        run_chunks<true>(a, c, st);
        if (l.taps > 1)
          hipLaunchKernelGGL(keep_inputs, dim3((channels + kPfThreads - 1) / kPfThreads), block, 0, st, b.qkv, l, channels, a->slot, a->flip, M);
      } else {
        const int keys = l.heads * l.head_dim;
        GemmArgs g = gemm_args(b.h, l.in_w, l.in_rows, D, l, EPI_GLA_IN);
        g.f0 = b.qkv; g.out = b.gate; g.out2 = b.low;
        launch_gemm<T, u16, T>(g, st);
        GemmArgs e = gemm_args(b.low, l.mid_w, keys, l.rank, l, EPI_GLA_DECAY);
        e.f0 = b.decay; e.ldo = keys;
        launch_gemm<T, u16, T>(e, st);
        c.qkv = b.qkv; c.values = b.qkv; c.value_ld = 2 * keys + W; c.value_at = 2 * keys;
        run_chunks<false>(a, c, st);
      }
      hipLaunchKernelGGL(state_out<T>, dim3((M * l.heads + 3) / 4), block, 0, st, b.o, b.gate, l, M, a->eps, b.mix);
    }
    GemmArgs o = gemm_args(b.mix, l.o_w, D, W, l, l.branches > 1 ? EPI_LOGITS : EPI_ADD);
    o.f0 = l.branches > 1 ? b.branch + l.branch * rows : b.x;
    launch_gemm<T, u16, T>(o, st);
    if (l.branch + 1 == l.branches) {
      const QmkHybridLayer& head = a->layers[i - l.branch];
      if (head.has_mlp) {
        GemmArgs g = gemm_args(b.h, head.mlp_w, 2 * head.ff, D, head, EPI_GEGLU);
        g.out = b.mix;
        launch_gemm<T, u16, T>(g, st);
        GemmArgs d = gemm_args(b.mix, head.down_w, D, head.ff, head, EPI_ADD);
        d.f0 = b.x;
        launch_gemm<T, u16, T>(d, st);
      }
    }
  }
  return hipGetLastError() == hipSuccess ? QMK_OK : QMK_ERR_LAUNCH;
}

}  // namespace hybrid
}  // namespace qmk

using namespace qmk;
using namespace qmk::hybrid;

extern "C" uint64_t qmk_hybrid_decode_bytes(const QmkHybridArgs* a) {
  if (check_shape(a) != QMK_OK || a->max_splits < 1 || a->max_splits > kMaxParts) return 0;
  DecodeBuffers b;
  return decode_buffers(a, nullptr, &b);
}

extern "C" uint64_t qmk_hybrid_prefill_bytes(const QmkHybridArgs* a) {
  if (check_shape(a) != QMK_OK || a->portion_rows < 1 || a->max_positions < 1) return 0;
  if (a->dtype == QMK_HYBRID_F32) {
    PrefillBuffers<float> b;
    return prefill_buffers<float>(a, nullptr, &b);
  }
  PrefillBuffers<u16> b;
  return prefill_buffers<u16>(a, nullptr, &b);
}

extern "C" int qmk_hybrid_prefill(const QmkHybridArgs* a) {
  if (a == nullptr) return QMK_ERR_NULL_ARG;
  if (int rc = check_launch(a, a->tokens); rc != QMK_OK) return rc;
  if (a->tokens > a->portion_rows || a->num_want < 0 || a->num_want > a->tokens) return QMK_ERR_SHAPE;
  if (a->num_want > 0 && (a->want == nullptr || a->logits == nullptr)) return QMK_ERR_NULL_ARG;
  return a->dtype == QMK_HYBRID_F32 ? prefill<float>(a) : prefill<u16>(a);
}

extern "C" int qmk_hybrid_decode_step(const QmkHybridArgs* a) {
  if (int rc = check_launch(a, 1); rc != QMK_OK) return rc;
  if (a->instructions == nullptr || a->barriers == nullptr || a->logits == nullptr) return QMK_ERR_NULL_ARG;
  if (a->num_queues < 1 || a->num_insts < 1 || a->barrier_groups < 1 || a->max_splits < 1 || a->max_splits > kMaxParts) return QMK_ERR_SHAPE;
  if (reinterpret_cast<uintptr_t>(a->barriers) % 128 != 0) return QMK_ERR_SHAPE;
  DecodeBuffers b;
  if (decode_buffers(a, a->workspace, &b) > a->workspace_bytes) return QMK_ERR_SCRATCH;
  DeviceInfo* dev = nullptr;
  if (int rc = device_info(&dev); rc != QMK_OK) return rc;
  if (a->num_queues > dev->max_queues) return QMK_ERR_TOO_MANY_QUEUES;
  DecodeParams p{};
  p.instructions = a->instructions; p.layers = a->layers_device; p.barriers = a->barriers; p.status = dev->status; p.timeline = a->timeline;
  p.candidates = b.candidates; p.embed = a->embed; p.head = a->head; p.final_norm = a->final_norm; p.token_in = a->token_in; p.token_out = a->token_out;
  p.logits = a->logits; p.u = b.u; p.x = b.x; p.out = b.out; p.proj = b.proj; p.mix = b.mix; p.absorbed = b.absorbed; p.part = b.part; p.ml = b.ml;
  p.num_insts = a->num_insts; p.num_layers = a->num_layers; p.groups = a->barrier_groups; p.width = a->width; p.width_true = a->width_true;
  p.streams = a->streams; p.vocab = a->vocab; p.vocab_rows = a->vocab_rows; p.slot = a->slot; p.position = a->position; p.flip = a->flip;
  p.max_splits = a->max_splits; p.eps = a->eps; p.logit_scale = a->logit_scale; p.logit_softcap = a->logit_softcap; p.spin_limit = a->spin_limit != 0 ? a->spin_limit : kDefaultSpinLimit;
  const hipStream_t st = static_cast<hipStream_t>(a->stream);
  auto launch = [&](auto kernel) { hipLaunchKernelGGL(kernel, dim3(a->num_queues), dim3(kThreads), 0, st, p); };
  const bool plain = a->streams == 0;
  if (a->dtype == QMK_HYBRID_F32) plain ? launch(decode_megakernel_hybrid<float, true>) : launch(decode_megakernel_hybrid<float, false>);
  else plain ? launch(decode_megakernel_hybrid<u16, true>) : launch(decode_megakernel_hybrid<u16, false>);
  return hipGetLastError() == hipSuccess ? QMK_OK : QMK_ERR_LAUNCH;
}

extern "C" int qmk_hybrid_status_fetch(void* stream, int32_t detail[4]) {
  DeviceInfo* dev = nullptr;
  if (int rc = device_info(&dev); rc != QMK_OK) return rc;
  if (hipStreamSynchronize(static_cast<hipStream_t>(stream)) != hipSuccess) return QMK_ERR_NO_DEVICE;
  int32_t host[kStatusWords] = {0};
  if (hipMemcpy(host, dev->status, sizeof(host), hipMemcpyDeviceToHost) != hipSuccess) return QMK_ERR_NO_DEVICE;
  if (detail != nullptr)
    for (int i = 0; i < 4; ++i) detail[i] = host[1 + i];
  if (host[0] != 0 && hipMemset(dev->status, 0, sizeof(host)) != hipSuccess) return QMK_ERR_NO_DEVICE;
  return host[0];
}

extern "C" int qmk_hybrid_max_queues(void) {
  DeviceInfo* dev = nullptr;
  return device_info(&dev) == QMK_OK ? dev->max_queues : -QMK_ERR_NO_DEVICE;
}

extern "C" int qmk_hybrid_abi_version(void) { return QMK_HYBRID_ABI_VERSION; }
