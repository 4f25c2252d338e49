// Prefill kernels of the hybrid route's plain residual: the residual and its norms, keys and values of the full attention,
// and the gated state recurrences (gated linear attention, gated delta rule) in chunks of sixteen tokens on the matrix cores.
//
// Recurrence of one head, state S [keys][values], decay g_t per key channel:
//   S <- g_t S,  u_t = beta_t (v_t - S^T k_t),  S <- S + k_t u_t^T,  o_t = S^T q_t        (gla: u_t = v_t)
// Over a chunk that starts from S, with G_t = g_1 .. g_t and D_ts = g_{s+1} .. g_t (products, never quotients: a decay may
// be small enough for its inverse to overflow):
//   X_t = (G_t k_t)^T S           u = T (v - X),  T = (I + diag(beta) A)^-1 diag(beta),  A_ts = sum_i k_t D_ts k_s  (s < t)
//   o_t = (G_t q_t)^T S + sum_{s <= t} B_ts u_s,  B_ts = sum_i q_t D_ts k_s
//   S  <- G_16 S + sum_s (D_16,s k_s) u_s^T
// chunk_prepare works out everything that no state enters, for all chunks at once; chunk_scan walks the chunks.
#pragma once

#include "qmk_hybrid_prefill.h"

namespace qmk {
namespace hybrid {

// Row m of the residual (row want[m] where given): x, or the token's embedding where x is not there yet, plus the normed
// outputs of two branches.  Leaves the sum in x (unless `want`), a copy in `dump`, and in h its norm, or [x; embedding].
struct ResidualArgs {
  float* x;
  const float *a, *b, *wa, *wb;   // branches, or NULL
  const u16* table;               // embedding
  const int64_t* tokens;
  const int32_t* want;
  const float* weight;            // of the norm; NULL: [x; embedding]
  float* dump;
  int embed, vocab, M, D, width, norm;
  float scale, eps;
};
template <class T>
__global__ __launch_bounds__(kPfThreads) void residual_rows(const ResidualArgs g, T* h) {
  __shared__ float scratch[4];
  const int D = g.D;
  int m = g.want != nullptr ? g.want[blockIdx.x] : blockIdx.x;
  m = m < 0 || m >= g.M ? 0 : m;
  long long token = g.tokens[m];
  if (token < 0 || token >= g.vocab) token = 0;
  const u16* e = g.table + token * D;
  float* x = g.x + static_cast<size_t>(m) * D;
  const float *a = g.a + static_cast<size_t>(m) * D, *b = g.b + static_cast<size_t>(m) * D;
  float sa = 0.f, sb = 0.f;
  const bool two = g.a != nullptr;
  if (two) {
    for (int i = threadIdx.x * 4; i < D; i += kPfThreads * 4) {
      const f32x4 u = read4(a + i), v = read4(b + i);
      sa += u[0] * u[0] + u[1] * u[1] + u[2] * u[2] + u[3] * u[3];
      sb += v[0] * v[0] + v[1] * v[1] + v[2] * v[2] + v[3] * v[3];
    }
    sa = g.scale / sqrtf(pf_block_sum(sa, scratch) / g.width + g.eps);
    sb = g.scale / sqrtf(pf_block_sum(sb, scratch) / g.width + g.eps);
  }
  auto value = [&](int i) {
    f32x4 v = g.embed ? read4(e + i) : read4(x + i);
    if (two) v += read4(a + i) * read4(g.wa + i) * sa + read4(b + i) * read4(g.wb + i) * sb;
    return v;
  };
  constexpr int kHeld = 4;
  f32x4 held[kHeld];
  float total = 0.f;
  auto take = [&](int i, f32x4 v) {
    total += v[0] + v[1] + v[2] + v[3];
    if (g.dump != nullptr) store4(g.dump + static_cast<size_t>(m) * D + i, v);
  };
#pragma unroll
  for (int j = 0; j < kHeld; ++j) {
    const int i = (j * kPfThreads + static_cast<int>(threadIdx.x)) * 4;
    held[j] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (i < D) take(i, held[j] = value(i));
  }
  for (int i = (kHeld * kPfThreads + threadIdx.x) * 4; i < D; i += kPfThreads * 4) take(i, value(i));
  T* out = h + static_cast<size_t>(blockIdx.x) * D * (g.weight == nullptr ? 2 : 1);
  float mean = 0.f, inv = 0.f;
  auto centred = [&](int i, f32x4 v) {
#pragma unroll
    for (int c = 0; c < 4; ++c) v[c] = i + c < g.width ? v[c] - mean : 0.f;
    return v;
  };
  if (g.weight != nullptr) {
    if (g.norm == QMK_NORM_LAYER) mean = pf_block_sum(total, scratch) / g.width;
    float sq = 0.f;
    auto add = [&](int i, f32x4 v) {
      v = centred(i, v);
      sq += v[0] * v[0] + v[1] * v[1] + v[2] * v[2] + v[3] * v[3];
    };
#pragma unroll
    for (int j = 0; j < kHeld; ++j) add((j * kPfThreads + threadIdx.x) * 4, held[j]);
    for (int i = (kHeld * kPfThreads + threadIdx.x) * 4; i < D; i += kPfThreads * 4) add(i, value(i));
    inv = 1.f / sqrtf(pf_block_sum(sq, scratch) / g.width + g.eps);
  }
  const bool keep = g.want == nullptr && (g.embed || two);
  auto put = [&](int i, f32x4 v) {
    if (keep) store4(x + i, v);
    if (g.weight != nullptr) {
      store4(out + i, centred(i, v) * inv * read4(g.weight + i));
    } else {
      store4(out + i, v);
      store4(out + D + i, read4(e + i));
    }
  };
#pragma unroll
  for (int j = 0; j < kHeld; ++j) {
    const int i = (j * kPfThreads + static_cast<int>(threadIdx.x)) * 4;
    if (i < D) put(i, held[j]);
  }
  for (int i = (kHeld * kPfThreads + threadIdx.x) * 4; i < D; i += kPfThreads * 4) put(i, value(i));
}

// v_t[key head][value][key] of keys 0 .. keys - 1 out of the cache: 64 keys x 64 columns a workgroup.
template <class T>
__global__ __launch_bounds__(kPfThreads) void transpose_values(const T* cache, int pitch, int row, int value_at, int v_dim, int keys, int cap, T* out) {
  __shared__ T tile[64][64 + 4 / sizeof(T)];
  const int key0 = blockIdx.x * 64, col0 = blockIdx.y * 64, kv = blockIdx.z;
  for (int id = threadIdx.x; id < 64 * 64; id += kPfThreads) {
    const int r = id >> 6, c = id & 63;
    if (key0 + r < keys && col0 + c < v_dim) tile[r][c] = cache[static_cast<size_t>(key0 + r) * pitch + kv * row + value_at + col0 + c];
  }
  __syncthreads();
  for (int id = threadIdx.x; id < 64 * 64; id += kPfThreads) {
    const int c = id >> 6, r = id & 63;
    if (key0 + r < keys && col0 + c < v_dim) out[(static_cast<size_t>(kv) * v_dim + col0 + c) * cap + key0 + r] = tile[r][c];
  }
}

constexpr int kChunkTokens = 16;
constexpr int kChunkWaves = 4;

// Tiles of sixteen key channels a wave of chunk_scan holds, and those of a head, the last ones zeros.
__host__ __device__ constexpr int wave_tiles(int head_dim) { return head_dim <= 64 ? 1 : head_dim <= 128 ? 2 : 4; }
__host__ __device__ constexpr int chunk_tiles(int head_dim) { return wave_tiles(head_dim) * kChunkWaves; }
// Floats of one (chunk, head): per tile the fragments of G q, G k and D k and the decays G over the whole chunk, then B and
// T.  A fragment is in the order the matrix instruction takes it: [lane][4].
__host__ __device__ constexpr int chunk_floats(int head_dim) { return chunk_tiles(head_dim) * (3 * 256 + 16) + 2 * 256; }

struct ChunkArgs {
  QmkHybridLayer layer;
  const float* qkv;      // [M][q, k, v]; delta: ahead of the convolution
  const float* decay;    // [M][heads * head_dim]
  const float* beta;     // delta: [M][beta_ld]
  float* chunks;         // [chunk][head][chunk_floats]
  float* values;         // [M][value_ld] at value_at; delta: written here
  float* out;            // [M][heads * v_dim]
  int M, beta_ld, value_ld, value_at, slot, flip;
};

// One workgroup per (chunk, head).  delta: convolution, silu and unit norm of the head's q and k, convolution and silu of its v.
template <bool DELTA>
__global__ __launch_bounds__(kPfThreads) void chunk_prepare(const ChunkArgs g) {
  constexpr int C = kChunkTokens;
  __shared__ float sq[C][kMaxHeadDim], sk[C][kMaxHeadDim], sg[C][kMaxHeadDim];
  __shared__ __align__(16) float sa[C][C], sb[C][C];
  __shared__ float step[C];
  const QmkHybridLayer& l = g.layer;
  const int dim = l.head_dim, n = l.v_dim, head = blockIdx.y, chunk = blockIdx.x, m0 = chunk * C, count = min(C, g.M - m0);
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int kv = head / (l.heads / l.kv_heads), keys = l.kv_heads * dim;

  // A thread takes a channel of q, k or v down the chunk's tokens.
  for (int id = tid; id < (DELTA ? 2 * dim + n : 2 * dim); id += kPfThreads) {
    const int part = id / dim < 2 ? id / dim : 2, c = id - part * dim;
    float v[C];
    if constexpr (DELTA) {
      const int W = conv_channels(l), taps = l.taps, ch = part == 0 ? kv * dim + c : part == 1 ? keys + kv * dim + c : 2 * keys + head * n + c;
      const float* x = g.qkv + ch;
      const float* old = l.shift + (static_cast<size_t>(g.slot) * 2 + g.flip) * (taps - 1) * W + ch;
      const float* weight = l.vec2 + ch;
      auto inside = [&](int at) { return x[static_cast<size_t>(min(at, g.M - 1)) * W]; };      // tokens behind the portion are not used
      auto input = [&](int at) { return at >= 0 ? inside(at) : old[static_cast<size_t>(at + taps - 1) * W]; };
      constexpr int kFew = 4;
      if (taps <= kFew) {
        float in[C + kFew - 1], w[kFew];
#pragma unroll
        for (int j = 0; j < kFew; ++j) w[j] = j >= kFew - taps ? weight[static_cast<size_t>(j - kFew + taps) * W] : 0.f;
#pragma unroll
        for (int j = 0; j < kFew - 1; ++j) in[j] = j >= kFew - taps ? input(m0 - (kFew - 1) + j) : 0.f;
#pragma unroll
        for (int j = 0; j < C; ++j) in[kFew - 1 + j] = inside(m0 + j);
#pragma unroll
        for (int t = 0; t < C; ++t) {
          v[t] = 0.f;
#pragma unroll
          for (int j = 0; j < kFew; ++j) v[t] = fmaf(w[j], in[t + j], v[t]);
        }
      } else {
#pragma unroll
        for (int t = 0; t < C; ++t) {
          v[t] = 0.f;
          for (int j = 0; j < taps; ++j) v[t] = fmaf(weight[static_cast<size_t>(j) * W], input(m0 + t - (taps - 1) + j), v[t]);
        }
      }
#pragma unroll
      for (int t = 0; t < C; ++t) v[t] *= sigmoid(v[t]);
      if (part == 2) {
        float* to = g.values + static_cast<size_t>(m0) * g.value_ld + g.value_at + head * n + c;
#pragma unroll
        for (int t = 0; t < C; ++t)
          if (t < count) to[static_cast<size_t>(t) * g.value_ld] = v[t];
        continue;
      }
    } else {
      const int ld = 2 * keys + l.heads * n;
      const float* row = g.qkv + static_cast<size_t>(m0) * ld + part * keys + kv * dim + c;
#pragma unroll
      for (int t = 0; t < C; ++t) v[t] = row[static_cast<size_t>(min(t, count - 1)) * ld] * (part == 0 ? l.q_scale : 1.f);
    }
    auto& to = part == 0 ? sq : sk;
#pragma unroll
    for (int t = 0; t < C; ++t) to[t][c] = t < count ? v[t] : 0.f;
  }
  if constexpr (DELTA) {
    if (tid < count) step[tid] = g.beta[static_cast<size_t>(m0 + tid) * g.beta_ld + head];
  }
  for (int c = tid; c < dim; c += kPfThreads) {
    const float* row = g.decay + static_cast<size_t>(m0) * l.heads * dim + head * dim + c;
    float v[C];
#pragma unroll
    for (int t = 0; t < C; ++t) v[t] = row[static_cast<size_t>(min(t, count - 1)) * l.heads * dim];
#pragma unroll
    for (int t = 0; t < C; ++t) sg[t][c] = t < count ? v[t] : 1.f;
  }
  __syncthreads();
  if constexpr (DELTA) {      // unit vectors
    for (int t = wave; t < C; t += kChunkWaves) {
      float nq = 0.f, nk = 0.f;
      for (int c = lane; c < dim; c += 64) {
        nq = fmaf(sq[t][c], sq[t][c], nq);
        nk = fmaf(sk[t][c], sk[t][c], nk);
      }
      const float iq = l.q_scale / sqrtf(wave_sum(nq) + 1e-6f), ik = 1.f / sqrtf(wave_sum(nk) + 1e-6f);
      for (int c = lane; c < dim; c += 64) {
        sq[t][c] *= iq;
        sk[t][c] *= ik;
      }
    }
    __syncthreads();
  }

  float* rec = g.chunks + (static_cast<size_t>(chunk) * l.heads + head) * chunk_floats(dim);
  const int tiles = dim / 16, stored = chunk_tiles(dim);
  float *rq = rec, *rk = rq + stored * 256, *rd = rk + stored * 256, *rg = rd + stored * 256, *rb = rg + stored * 16, *rt = rb + 256;
  for (int i = tiles * 256 + tid; i < stored * 256; i += kPfThreads) rq[i] = rk[i] = rd[i] = 0.f;
  if (tid >= dim && tid < stored * 16) rg[tid] = 0.f;
  if (tid < dim) {
    const int tile = tid >> 4, c = tid & 15;
    float cum = 1.f;
#pragma unroll
    for (int t = 0; t < C; ++t) {
      cum *= sg[t][tid];
      const int at = tile * 256 + ((c >> 2) * 16 + t) * 4 + (c & 3);
      rq[at] = sq[t][tid] * cum;
      if constexpr (DELTA) rk[at] = sk[t][tid] * cum;
    }
    rg[tid] = cum;
    float rest = 1.f;
#pragma unroll
    for (int t = C - 1; t >= 0; --t) {
      rd[tile * 256 + ((t >> 2) * 16 + c) * 4 + (t & 3)] = sk[t][tid] * rest;
      rest *= sg[t][tid];
    }
  }
  // Pairs: sixteen lanes share an s, channels 16 apart each; the decayed key runs down the tokens.
  {
    const int s = tid >> 4, part = tid & 15;
    float run[kMaxHeadDim / 16];
#pragma unroll
    for (int j = 0; j < kMaxHeadDim / 16; ++j) run[j] = 0.f;
    for (int t = 0; t < C; ++t) {
      float da = 0.f, db = 0.f;
#pragma unroll
      for (int j = 0; j < kMaxHeadDim / 16; ++j) {
        if (j < tiles) {
          const int c = j * 16 + part;
          const float kt = sk[t][c];
          run[j] *= sg[t][c];
          da = fmaf(kt, run[j], da);
          if (t == s) run[j] = kt;
          db = fmaf(sq[t][c], run[j], db);
        }
      }
      auto sum16 = [](float v) {
        v += dpp_f32<kDppQuadXor1>(0.f, v);
        v += dpp_f32<kDppQuadXor2>(0.f, v);
        v += dpp_f32<0x124>(0.f, v);        // row_ror:4
        v += dpp_f32<0x128>(0.f, v);        // row_ror:8
        return v;
      };
      db = sum16(db);
      if constexpr (DELTA) da = sum16(da);
      if (part == 0) {
        sb[t][s] = db;                       // zero above the diagonal
        sa[t][s] = da;                       // ... and on it
      }
    }
  }
  __syncthreads();
  if (tid < 256) rb[tid] = sb[(tid >> 2) & 15][(tid >> 6) * 4 + (tid & 3)];
  if constexpr (DELTA) {
    if (tid < C) {     // column tid of T
      float col[C];
#pragma unroll
      for (int t = 0; t < C; ++t) {
        float acc = t == tid ? 1.f : 0.f;
#pragma unroll
        for (int j = 0; j < t; ++j) acc = fmaf(-sa[t][j], col[j], acc);
        col[t] = t < count ? acc * step[t] : 0.f;
        rt[((tid >> 2) * 16 + t) * 4 + (tid & 3)] = col[t];
      }
    }
  }
}

// The convolution's last inputs of a portion, for the next one.
__global__ __launch_bounds__(kPfThreads) void keep_inputs(const float* x, QmkHybridLayer l, int W, int slot, int flip, int M) {
  const int c = blockIdx.x * kPfThreads + threadIdx.x, n = l.taps - 1;
  if (c >= W) return;
  const float* old = l.shift + (static_cast<size_t>(slot) * 2 + flip) * n * W;
  float* now = l.shift + (static_cast<size_t>(slot) * 2 + 1 - flip) * n * W;
  for (int j = 0; j < n; ++j) {
    const int t = M - n + j;
    now[static_cast<size_t>(j) * W + c] = t >= 0 ? x[static_cast<size_t>(t) * W + c] : old[static_cast<size_t>(t + n) * W + c];
  }
}

// One head and sixteen value columns a workgroup; a wave holds TILES tiles of sixteen key channels of the state as the
// accumulators of the matrix instruction, which are also the second operand of the products that read it.  Tiles behind the
// last one are zeros and take part: with a branch around each tile's products this compiler has left out the wait between a
// tile's last product and the first use of its result on the path that skips the next tile.  Loads have no branches either,
// so that kAhead chunks are in flight: a chunk, or token, behind the last one is the last one again, and its value is either
// not used or multiplied by zero.
template <int TILES, bool DELTA>
__global__ __launch_bounds__(kChunkWaves * 64) void chunk_scan(const ChunkArgs g) {
  constexpr int kAhead = TILES <= 2 ? 4 : 2;      // chunks in flight
  __shared__ f32x4 px[2][kChunkWaves][64], po[2][kChunkWaves][64];
  const QmkHybridLayer& l = g.layer;
  const int dim = l.head_dim, n = l.v_dim, head = blockIdx.x, v0 = blockIdx.y * 16;
  constexpr int tiles = TILES * kChunkWaves;
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), col = lane & 15, quad = lane >> 4;
  const int tile0 = wave * TILES, mine = min(max(dim / 16 - tile0, 0), TILES);
  const int chunks = (g.M + kChunkTokens - 1) / kChunkTokens;
  const size_t step = static_cast<size_t>(l.heads) * chunk_floats(dim);
  const float* rec = g.chunks + static_cast<size_t>(head) * chunk_floats(dim);
  float* state = l.state + (static_cast<size_t>(g.slot) * l.heads + head) * dim * n + v0 + col;
  const float* values = g.values + g.value_at + head * n + v0 + col;
  f32x4 s[TILES];
#pragma unroll
  for (int j = 0; j < TILES; ++j)
#pragma unroll
    for (int i = 0; i < 4; ++i) s[j][i] = j < mine ? state[static_cast<size_t>((tile0 + j) * 16 + quad * 4 + i) * n] : 0.f;

  struct Fragments {
    f32x4 q[TILES], k[TILES], d[TILES], g[TILES], b, t, v;
  };
  auto fetch = [&](Fragments& f, int chunk) {
    chunk = min(chunk, chunks - 1);
    const float* r = rec + chunk * step;
#pragma unroll
    for (int j = 0; j < TILES; ++j) {
      const int at = (tile0 + j) * 256 + lane * 4;
      if constexpr (DELTA) f.k[j] = read4(r + tiles * 256 + at);
      f.q[j] = read4(r + at);
      f.d[j] = read4(r + tiles * 512 + at);
      f.g[j] = read4(r + tiles * 768 + (tile0 + j) * 16 + quad * 4);
    }
    f.b = read4(r + tiles * 784 + lane * 4);
    if constexpr (DELTA) f.t = read4(r + tiles * 784 + 256 + lane * 4);
#pragma unroll
    for (int i = 0; i < 4; ++i) f.v[i] = values[static_cast<size_t>(min(chunk * kChunkTokens + quad * 4 + i, g.M - 1)) * g.value_ld];
  };
  auto product = [](f32x4 a, f32x4 b, f32x4 c) {
#pragma unroll
    for (int i = 0; i < 4; ++i) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a[i], b[i], c, 0, 0, 0);
    return c;
  };
  auto advance = [&](const Fragments& f, int chunk) {
    const int buf = chunk & 1;
    f32x4 x = {}, o = {};
    if constexpr (DELTA) {
#pragma unroll
      for (int j = 0; j < TILES; ++j) x = product(f.k[j], s[j], x);
      px[buf][wave][lane] = x;
    }
#pragma unroll
    for (int j = 0; j < TILES; ++j) o = product(f.q[j], s[j], o);
    po[buf][wave][lane] = o;
    __syncthreads();
    f32x4 u = f.v;
    if constexpr (DELTA) {
#pragma unroll
      for (int w = 0; w < kChunkWaves; ++w) u -= px[buf][w][lane];
      u = product(f.t, u, f32x4{0.f, 0.f, 0.f, 0.f});
    }
#pragma unroll
    for (int j = 0; j < TILES; ++j) s[j] = product(f.d[j], u, s[j] * f.g[j]);
    if (wave == (chunk & (kChunkWaves - 1))) {
      o = product(f.b, u, f32x4{0.f, 0.f, 0.f, 0.f});
#pragma unroll
      for (int w = 0; w < kChunkWaves; ++w) o += po[buf][w][lane];
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        const int m = chunk * kChunkTokens + quad * 4 + i;
        if (m < g.M) g.out[static_cast<size_t>(m) * l.heads * n + head * n + v0 + col] = o[i];
      }
    }
  };
  Fragments f[kAhead];
#pragma unroll
  for (int a = 0; a < kAhead; ++a) fetch(f[a], a);
  int chunk = 0;
  for (; chunk + kAhead <= chunks; chunk += kAhead) {
#pragma unroll
    for (int a = 0; a < kAhead; ++a) {
      advance(f[a], chunk + a);
      fetch(f[a], chunk + a + kAhead);
    }
  }
#pragma unroll
  for (int a = 0; a < kAhead - 1; ++a)
    if (chunk + a < chunks) advance(f[a], chunk + a);
#pragma unroll
  for (int j = 0; j < TILES; ++j)
    if (j < mine)
#pragma unroll
      for (int i = 0; i < 4; ++i) state[static_cast<size_t>((tile0 + j) * 16 + quad * 4 + i) * n] = s[j][i];
}

// Per-head norm, weight and gate behind the recurrence: one wave per (token, head).
template <class T>
__global__ __launch_bounds__(kPfThreads) void state_out(const float* o, const T* gate, QmkHybridLayer l, int M, float eps, T* out) {
  const int id = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (id >= M * l.heads) return;
  const int n = l.v_dim;
  const size_t at = static_cast<size_t>(id) * n;
  float sq = 0.f;
  for (int i = lane; i < n; i += 64) sq = fmaf(o[at + i], o[at + i], sq);
  const float inv = 1.f / sqrtf(wave_sum(sq) / l.v_true + eps);
  for (int i = lane; i < n; i += 64) out[at + i] = from_f32<T>(o[at + i] * inv * l.vec0[i] * to_f32(gate[at + i]));
}

}  // namespace hybrid
}  // namespace qmk
