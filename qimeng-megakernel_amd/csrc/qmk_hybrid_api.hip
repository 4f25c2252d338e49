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

template <class T>
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
        case OP_LM_HEAD: ok = op_rows<T>(p, s, o); break;
        case OP_LATENT_ATTEND: ok = op_latent_attend<T>(p, s, o); break;
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
    int a = 0, b = 0;
    void* sym = nullptr;
    if (hipGetDeviceProperties(&prop, dev) != hipSuccess ||
        hipOccupancyMaxActiveBlocksPerMultiprocessor(&a, decode_megakernel_hybrid<u16>, kThreads, 0) != hipSuccess ||
        hipOccupancyMaxActiveBlocksPerMultiprocessor(&b, decode_megakernel_hybrid<float>, kThreads, 0) != hipSuccess ||
        hipGetSymbolAddress(&sym, HIP_SYMBOL(g_status)) != hipSuccess || hipMemset(sym, 0, sizeof(int32_t) * kStatusWords) != hipSuccess)
      return QMK_ERR_NO_DEVICE;
    d.max_queues = std::min(std::min(a, b) * prop.multiProcessorCount, kMaxQueues);
    d.status = static_cast<int32_t*>(sym);
    d.ready = true;
  }
  *out = &d;
  return QMK_OK;
}

inline size_t align_up(size_t n) { return (n + 255) & ~size_t(255); }
inline bool m16(int v) { return v > 0 && v % 16 == 0; }
inline int element(const QmkHybridArgs* a) { return a->dtype == QMK_HYBRID_F32 ? 4 : 2; }

bool layer_ok(const QmkHybridArgs* a, const QmkHybridLayer& l) {
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
    default: return false;
  }
}

int check_shape(const QmkHybridArgs* a) {
  if (a == nullptr || a->layers == nullptr) return QMK_ERR_NULL_ARG;
  if (a->struct_size != sizeof(QmkHybridArgs)) return QMK_ERR_ABI;
  if (a->dtype > QMK_HYBRID_F32) return QMK_ERR_MODEL;
  if (a->num_layers < 1 || !m16(a->width) || a->width > kMaxK || a->width_true < 1 || a->width_true > a->width || a->streams < 1 ||
      a->streams > kMaxStreams || a->vocab < 1 || !m16(a->vocab_rows) || a->vocab > a->vocab_rows || !(a->eps >= 0.f))
    return QMK_ERR_SHAPE;
  for (int i = 0; i < a->num_layers; ++i)
    if (!layer_ok(a, a->layers[i])) return QMK_ERR_SHAPE;
  return QMK_OK;
}

bool layer_pointers(const QmkHybridLayer& l) {
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
    if (l.type == QMK_MIXER_LATENT && l.ring < std::min(a->position + tokens, l.window - 1 + tokens)) return QMK_ERR_SHAPE;
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
  float *u, *x, *proj, *mix, *absorbed, *part, *ml;
};
size_t decode_buffers(const QmkHybridArgs* a, void* base, DecodeBuffers* b) {
  size_t proj = 0, mix = 0, absorbed = 0, part = 0, ml = 0;
  for (int i = 0; i < a->num_layers; ++i) {
    const QmkHybridLayer& l = a->layers[i];
    proj = std::max<size_t>(proj, l.in_rows);
    mix = std::max<size_t>(mix, std::max(l.mix_width, l.has_mlp ? l.ff : 0));
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
  b->x = c.take<float>(static_cast<size_t>(a->streams) * a->width);
  b->proj = c.take<float>(proj);
  b->mix = c.take<float>(mix);
  b->absorbed = c.take<float>(absorbed);
  b->part = c.take<float>(part);
  b->ml = c.take<float>(ml);
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

template <class T, int QT, int VT>
void launch_attention(const QmkHybridArgs* a, const QmkHybridLayer& l, const PrefillBuffers<T>& b, int first, int cap, hipStream_t st) {
  hipLaunchKernelGGL((window_attention<T, QT, VT>), dim3((a->tokens + 63) / 64, l.heads), dim3(kPfThreads), 0, st, b.p0, b.kn, b.rows, b.vt, b.p1, l,
                     first, a->position, a->tokens, cap, b.mix);
}

template <class T>
int prefill(const QmkHybridArgs* a) {
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
      if (l.q_stride <= 128 && l.v_dim <= 64) launch_attention<T, 4, 4>(a, l, b, first, cap, st);
      else if (l.q_stride <= 192 && l.v_dim <= 128) launch_attention<T, 6, 8>(a, l, b, first, cap, st);
      else launch_attention<T, 8, 16>(a, l, b, first, cap, st);
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
  p.logits = a->logits; p.u = b.u; p.x = b.x; p.proj = b.proj; p.mix = b.mix; p.absorbed = b.absorbed; p.part = b.part; p.ml = b.ml;
  p.num_insts = a->num_insts; p.num_layers = a->num_layers; p.groups = a->barrier_groups; p.width = a->width; p.width_true = a->width_true;
  p.streams = a->streams; p.vocab = a->vocab; p.vocab_rows = a->vocab_rows; p.slot = a->slot; p.position = a->position; p.flip = a->flip;
  p.max_splits = a->max_splits; p.eps = a->eps; p.spin_limit = a->spin_limit != 0 ? a->spin_limit : kDefaultSpinLimit;
  const hipStream_t st = static_cast<hipStream_t>(a->stream);
  if (a->dtype == QMK_HYBRID_F32) hipLaunchKernelGGL(decode_megakernel_hybrid<float>, dim3(a->num_queues), dim3(kThreads), 0, st, p);
  else hipLaunchKernelGGL(decode_megakernel_hybrid<u16>, dim3(a->num_queues), dim3(kThreads), 0, st, p);
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
