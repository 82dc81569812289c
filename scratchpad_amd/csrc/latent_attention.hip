// Attention over a compressed (latent) key/value cache.  Per token the pool holds ONE row [c | k_rot]: the normed
// latent c (rank C) from which every head's unrotated key W_uk c and value W_uv c derive, and the rotated key part
// (R dimensions) all heads share.  The up-projections are folded into the query and the output:
//   score(t, s, h) = (W_uk_h^T q_h[t]) . c[s] + q_rot_h[t] . k_rot[s]          out_h[t] = W_uv_h (sum_s p(t, s, h) c[s])
// so the kernel is multi-query attention with key width C + R and value width C over the pool's rows; the two per-head
// products around it are sp_head_linear (out[t, h] = W_h x[t, h], optionally times sigmoid(gate)).
//
// Rotation: interleaved pairs (2i, 2i+1), angle = position * frequency[i] in fp32, cos and sin scaled by `mag`
// (frequency table and magnitude are the caller's: plain, or YaRN-blended).  The store can rotate the query's rotated part in
// the same launch; a layer that reads another layer's rows only rotates its query.
#include "seq_batch.h"

namespace sp {
namespace {

// in place on x[t, h, offset + 0 .. R) for every head
template <typename Tag>
__global__ void rotary_interleaved_kernel(void* x, const int64_t* positions, const float* freq, float mag, int H, int R,
                                          int64_t token_stride, int64_t head_stride, int offset) {
  typedef Elem<Tag> E;
  const int64_t t = blockIdx.x;
  const float pos = (float)positions[t];
  const int half = R / 2;
  for (int e = threadIdx.x; e < H * half; e += blockDim.x) {
    const int h = e / half, i = e % half;
    const float a = pos * freq[i];
    const float c = cosf(a) * mag, s = sinf(a) * mag;
    const int64_t at = t * token_stride + (int64_t)h * head_stride + offset + 2 * i;
    const float u = E::load(x, at), v = E::load(x, at + 1);
    E::store(x, at, u * c - v * s);
    E::store(x, at + 1, v * c + u * s);
  }
}

// pool[loc[t]] = [ rmsnorm(dkv[t, :C]) * w | rotate(dkv[t, C:C+R]) ]   (the first rot_dims of the R rotate, the rest pass);
// q (optional): q[t, h, q_offset .. q_offset + rot_dims) rotated in place for every head.  The token's cosines and sines
// (times mag) wait in LDS for all its heads.
constexpr int kMaxRot = 512;
template <typename Tag>
__global__ void __launch_bounds__(kBlock)
latent_kv_store_kernel(void* pool, int64_t pool_stride, const void* dkv, int64_t dkv_stride, const float* norm_w, void* q,
                       int64_t q_stride, int64_t q_head_stride, int q_offset, int H, const int64_t* positions,
                       const float* freq, float mag, const int64_t* loc, int C, int R, int rot_dims, float eps) {
  typedef Elem<Tag> E;
  __shared__ float red[kBlock / 64];
  __shared__ float cosine[kMaxRot / 2], sine[kMaxRot / 2];
  const int64_t t = blockIdx.x;
  const int half = rot_dims / 2;
  const float pos = (float)positions[t];
  for (int i = threadIdx.x; i < half; i += blockDim.x) {
    const float a = pos * freq[i];
    cosine[i] = cosf(a) * mag;
    sine[i] = sinf(a) * mag;
  }
  __syncthreads();
  if (q)
    for (int e = threadIdx.x; e < H * half; e += blockDim.x) {
      const int h = e / half, i = e % half;
      const int64_t at = t * q_stride + (int64_t)h * q_head_stride + q_offset + 2 * i;
      const float u = E::load(q, at), v = E::load(q, at + 1);
      E::store(q, at, u * cosine[i] - v * sine[i]);
      E::store(q, at + 1, v * cosine[i] + u * sine[i]);
    }
  if (!pool) return;
  const int64_t src = t * dkv_stride, dst = loc[t] * pool_stride;
  float ss = 0.f;
  for (int i = threadIdx.x; i < C; i += blockDim.x) {
    const float v = E::load(dkv, src + i);
    ss += v * v;
  }
  ss = block_sum(ss, red);
  const float inv = 1.f / sqrtf(ss / (float)C + eps);
  for (int i = threadIdx.x; i < C; i += blockDim.x) E::store(pool, dst + i, E::load(dkv, src + i) * inv * norm_w[i]);
  for (int i = threadIdx.x; i < half; i += blockDim.x) {
    const float u = E::load(dkv, src + C + 2 * i), v = E::load(dkv, src + C + 2 * i + 1);
    E::store(pool, dst + C + 2 * i, u * cosine[i] - v * sine[i]);
    E::store(pool, dst + C + 2 * i + 1, v * cosine[i] + u * sine[i]);
  }
  for (int i = rot_dims + threadIdx.x; i < R; i += blockDim.x) E::store(pool, dst + C + i, E::load(dkv, src + C + i));
}

constexpr int kMaxPerLane = 16;      // value width C <= 64 * kMaxPerLane

// One wave per (token, head); 4 heads of a token per workgroup.  Keys in tiles of 64: lane = key for the scores,
// lane = value channel for the weighted sum; running maximum and sum in fp32.
template <typename Tag>
__global__ void __launch_bounds__(256)
latent_attention_kernel(void* out, const void* q_lat, int64_t lat_token_stride, int64_t lat_head_stride, const void* q_rot,
                        const void* pool, int64_t pool_stride, const int32_t* req_to_token, int64_t table_stride, SeqBatch s,
                        int64_t T, int H, int C, int R, int64_t qrot_token_stride, int64_t qrot_head_stride, float scale) {
  typedef Elem<Tag> E;
  extern __shared__ float smem[];
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  const int64_t t = blockIdx.x;
  const int h = blockIdx.y * 4 + wave;
  if (h >= H) return;                                    // (no workgroup barrier below)
  float* sq = smem + (size_t)wave * (C + R + 64);        // this wave's query [C + R], then its 64 weights
  float* sp_ = sq + C + R;
  int b;
  int64_t start, prefix;
  seq_of_token(s, t, b, start, prefix);
  const int64_t keys = prefix + (t - start) + 1;        // positions 0 .. own
  const int32_t* table = req_to_token + load_idx(s.req_pool_indices, b, s.idx64) * table_stride;
  for (int i = lane; i < C; i += 64) sq[i] = E::load(q_lat, t * lat_token_stride + h * lat_head_stride + i) * scale;
  for (int i = lane; i < R; i += 64) sq[C + i] = E::load(q_rot, t * qrot_token_stride + (int64_t)h * qrot_head_stride + i) * scale;
  __builtin_amdgcn_wave_barrier();
  float m = -INFINITY, l = 0.f;
  float acc[kMaxPerLane];
#pragma unroll
  for (int i = 0; i < kMaxPerLane; ++i) acc[i] = 0.f;
  const int W = C + R;
  for (int64_t k0 = 0; k0 < keys; k0 += 64) {
    const int n = (int)(keys - k0 < 64 ? keys - k0 : 64);
    float sc = -INFINITY;
    int64_t row = 0;
    if (lane < n) {
      row = (int64_t)table[k0 + lane] * pool_stride;
      float d = 0.f;
      for (int i = 0; i < W; ++i) d += sq[i] * E::load(pool, row + i);
      sc = d;
    }
    float tm = sc;
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) tm = fmaxf(tm, __shfl_xor(tm, off, 64));
    const float m_new = fmaxf(m, tm);
    const float corr = expf(m - m_new);                 // first tile: exp(-inf) = 0
    const float p = lane < n ? expf(sc - m_new) : 0.f;
    l = l * corr + wave_sum(p);
    m = m_new;
    sp_[lane] = p;
    __builtin_amdgcn_wave_barrier();
#pragma unroll
    for (int i = 0; i < kMaxPerLane; ++i) acc[i] *= corr;
    for (int j = 0; j < n; ++j) {
      const int64_t rj = (int64_t)table[k0 + j] * pool_stride;
      const float pj = sp_[j];
#pragma unroll
      for (int i = 0; i < kMaxPerLane; ++i) {
        const int c = lane + 64 * i;
        if (c < C) acc[i] += pj * E::load(pool, rj + c);
      }
    }
    __builtin_amdgcn_wave_barrier();
  }
  const float inv = 1.f / l;
#pragma unroll
  for (int i = 0; i < kMaxPerLane; ++i) {
    const int c = lane + 64 * i;
    if (c < C) E::store(out, t * lat_token_stride + h * lat_head_stride + c, acc[i] * inv);
  }
}

// ---- the same attention on the matrix cores, for 16-bit types -------------------------------------------------------
// All heads of a token read the same pool rows, so the queries of one request are ONE list of rows (token-major, then head)
// whatever the head count.  A workgroup of NW waves takes RB blocks of 16 such rows and walks the keys they can see in tiles
// of 64, staged in LDS row by row (the next tile's rows are in flight during the work on this one):
//   S^T = K Q^T   v_mfma_f32_16x16x32, first operand = 16 key rows from LDS, second = the query fragments, in registers for
//                 the whole walk (rows too wide for that: the later steps' fragments wait in LDS): wave w forms KBW of the
//                 tile's 4 key blocks for RBW of the RB row blocks.  A lane receives four keys of ONE query; a query's maximum is a reduction over its lanes and, through LDS, over the waves.
//   P             exp of the scores, as a 16-bit value plus its 16-bit remainder (the weights are never rounded to 8 bits
//                 of mantissa), goes to LDS in exactly the register layout the second product wants.
//   O^T = V^T P^T the value is the first C columns of the same rows: its transposed fragments come from the key tile by
//                 transposing LDS reads.  Wave w owns the value channels [16 DTW w, 16 DTW (w + 1)) of all RB row blocks.
// Two waves per SIMD (NW = 8) where there are rows enough: one's softmax runs under the other's matrix instructions.
// With splits > 1 the tiles of a row block are shared out over blockIdx.y; every share writes its unnormalised sum, maximum
// and denominator, and latent_merge_kernel joins them in the order of the keys (decode steps: few rows, many keys).
typedef float f32x4_l __attribute__((ext_vector_type(4)));
typedef __bf16 bf16x8_l __attribute__((ext_vector_type(8)));
typedef _Float16 f16x8_l __attribute__((ext_vector_type(8)));
typedef short s16x4_l __attribute__((ext_vector_type(4)));
template <typename Tag>
__device__ __forceinline__ f32x4_l mfma_l(const u32x4& a, const u32x4& b, const f32x4_l& c);
template <>
__device__ __forceinline__ f32x4_l mfma_l<bf16_tag>(const u32x4& a, const u32x4& b, const f32x4_l& c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8_l, a), __builtin_bit_cast(bf16x8_l, b), c, 0, 0, 0);
}
template <>
__device__ __forceinline__ f32x4_l mfma_l<f16_tag>(const u32x4& a, const u32x4& b, const f32x4_l& c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_f16(__builtin_bit_cast(f16x8_l, a), __builtin_bit_cast(f16x8_l, b), c, 0, 0, 0);
}

struct LatentArgs {
  void* out;
  const void* q_lat;
  const void* q_rot;
  const void* pool;
  const int32_t* req_to_token;
  float* part;                 // splits > 1: [splits][T * H][C] sums, then [splits][T * H][2] maximum and denominator
  int64_t lat_token_stride, lat_head_stride, qrot_token_stride, qrot_head_stride, pool_stride, table_stride, T;
  int H, C, R, splits;
  float scale;
};

constexpr int kKeyTile = 64;
constexpr int kMaxSplits = 64;
constexpr float kSlack = 10.f;                       // in powers of two
template <int KS>
constexpr int key_row() { return 32 * KS + 8; }      // elements per LDS row: 16 bytes of padding spread the rows over the banks
template <int KS, int RB>
constexpr int query_steps() { return KS > 10 && RB > 1 ? (RB > 2 ? 4 : KS / 3) : KS; }      // steps whose query fragments stay in registers
template <int KS, int RB, int NW>
constexpr size_t latent_lds() {
  return (size_t)kKeyTile * key_row<KS>() * 2 + (size_t)RB * 4096 + (size_t)RB * (KS - query_steps<KS, RB>()) * 1024 +
         (NW * 2 * 16 + RB * 16 + NW * 2 * 16 + kKeyTile) * 4;
}

template <typename Tag, int KS, int DTW, int RB, int NW>
__global__ void __launch_bounds__(64 * NW, NW / 4) latent_mfma_kernel(LatentArgs a, SeqBatch s) {
  typedef Elem<Tag> E;
  constexpr int RBW = RB > 1 ? 2 : 1;                 // row blocks a wave scores
  constexpr int GROUPS = RB / RBW;                    // groups of row blocks
  constexpr int KBW = 4 * GROUPS / NW;                // key blocks (of 4) a wave scores: GROUPS * (4 / KBW) = NW waves
  static_assert(KBW >= 1 && KBW * NW == 4 * GROUPS, "every key block of every row block has one wave");
  constexpr int KR = key_row<KS>();
  extern __shared__ __attribute__((aligned(16))) char lds[];
  uint16_t* sk = (uint16_t*)lds;                                       // [64][KR]
  u32x2* sp_ = (u32x2*)(lds + (size_t)kKeyTile * KR * 2);              // [RB][2][4 key blocks][64 lanes]
  constexpr int KQ = query_steps<KS, RB>();
  u32x4* sqf = (u32x4*)(lds + (size_t)kKeyTile * KR * 2 + RB * 4096);  // [RB][KS - KQ][64 lanes]
  float* smax = (float*)(sqf + RB * (KS - KQ) * 64);                   // [NW][RBW][16]
  float* scorr = smax + NW * 2 * 16;                                   // [RB][16]
  float* ssum = scorr + RB * 16;                                       // [NW][RBW][16]
  int32_t* sslot = (int32_t*)(ssum + NW * 2 * 16);                     // [64] pool rows of the next tile's keys
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, r16 = lane & 15, qd = lane >> 4;
  const int rg = wave % GROUPS, kg = wave / GROUPS;
  // which request and which of its row tiles
  int64_t start, len, prefix;
  int tile = blockIdx.x, b = 0;
  if (s.extend_seq_lens) {
    for (; b < s.B; ++b) {
      const int tiles = (int)(((int64_t)s.extend_seq_lens[b] * a.H + 16 * RB - 1) / (16 * RB));
      if (tile < tiles) {
        tile = tiles - 1 - tile;                                       // the tiles with most keys start first
        break;
      }
      tile -= tiles;
    }
    if (b >= s.B) return;
  } else {
    const int tiles = (a.H + 16 * RB - 1) / (16 * RB);
    b = tile / tiles;
    tile = tile % tiles;
    if (b >= s.B) return;
  }
  seq_span(s, b, start, len, prefix);
  const int64_t row0 = (int64_t)tile * 16 * RB, rows = len * a.H;      // rows of this request, this tile's first
  const int64_t last_row = row0 + 16 * RB <= rows ? row0 + 16 * RB - 1 : rows - 1;
  const int64_t keys = prefix + last_row / a.H + 1;
  const int64_t tiles_k = (keys + kKeyTile - 1) / kKeyTile;
  const float scale2 = a.scale * 1.4426950408889634f;                  // scores in powers of two
  const int64_t per = (tiles_k + a.splits - 1) / a.splits;
  const int64_t kt0 = (int64_t)blockIdx.y * per, kt1 = kt0 + per < tiles_k ? kt0 + per : tiles_k;
  const int32_t* table = a.req_to_token + load_idx(s.req_pool_indices, b, s.idx64) * a.table_stride;
  const int chunks = (a.C + a.R) / 8;                                  // 16-byte pieces of a pool row
  // this lane's query rows (column r16 of every S^T block): fragments and the last key each may see
  u32x4 qf[RBW][KQ];
  int64_t qpos[RBW];
#pragma unroll
  for (int i = 0; i < RBW; ++i) {
    const int64_t r = row0 + 16 * (rg * RBW + i) + r16;
    const bool on = r < rows;
    const int64_t t = start + (on ? r / a.H : 0), h = on ? r % a.H : 0;
    qpos[i] = on ? prefix + (t - start) : -1;
#pragma unroll
    for (int st = 0; st < KS; ++st) {
      const int k = 32 * st + 8 * qd;
      u32x4 f = {0u, 0u, 0u, 0u};
      if (on && k < a.C) f = ld16((const char*)a.q_lat + (t * a.lat_token_stride + h * a.lat_head_stride + k) * 2);
      else if (on && k < a.C + a.R) f = ld16((const char*)a.q_rot + (t * a.qrot_token_stride + h * a.qrot_head_stride + k - a.C) * 2);
      if (st < KQ) qf[i][st < KQ ? st : 0] = f;
      else if (kg == 0) sqf[((rg * RBW + i) * (KS - KQ) + st - KQ) * 64 + lane] = f;      // (read behind the walk's barriers)
    }
  }
  f32x4_l oacc[DTW][RB];
#pragma unroll
  for (int d = 0; d < DTW; ++d)
#pragma unroll
    for (int i = 0; i < RB; ++i) oacc[d][i] = f32x4_l{0.f, 0.f, 0.f, 0.f};
  float m[RBW], l[RBW];
#pragma unroll
  for (int i = 0; i < RBW; ++i) {
    m[i] = -INFINITY;
    l[i] = 0.f;
  }
  // a thread moves ONE 16-byte column of the rows key_first, key_first + KPP, ... of every tile: its addresses differ by
  // constants.  Keys behind the last one and columns behind the row repeat the last of them - finite numbers that meet a zero
  // weight or a zero of the query - so that no load waits for a branch
  constexpr int CW = 4 * KS, KPP = 64 * NW / CW, NP = (kKeyTile + KPP - 1) / KPP;
  const int key_first = threadIdx.x / CW, c = threadIdx.x % CW;
  const bool mover = key_first < KPP;
  const char* column = (const char*)a.pool + 16 * (c < chunks ? c : chunks - 1);
  u32x4 stage[NP];
  auto fetch = [&]() {                                                 // from the slots in LDS, behind a barrier
    constexpr int PART = 6;                                            // addresses formed at a time
#pragma unroll
    for (int u0 = 0; u0 < NP; u0 += PART) {
      int32_t row[PART];
#pragma unroll
      for (int u = u0; u < NP && u < u0 + PART; ++u)
        row[u - u0] = sslot[key_first + u * KPP < kKeyTile ? key_first + u * KPP : kKeyTile - 1];
#pragma unroll
      for (int u = u0; u < NP && u < u0 + PART; ++u) stage[u] = ld16(column + (int64_t)row[u - u0] * (2 * a.pool_stride));
      __builtin_amdgcn_sched_barrier(0);
    }
  };
  auto slot_of = [&](int64_t kt) {                                     // the slot of a tile's key (threads 0 .. 63 use it)
    const int64_t kk = kt * kKeyTile + (threadIdx.x & 63);
    return table[kk < keys ? kk : keys - 1];
  };
  int32_t slot = slot_of(kt0);
  if (threadIdx.x < kKeyTile) sslot[threadIdx.x] = slot;
  __syncthreads();
  if (kt0 < kt1) fetch();
  slot = slot_of(kt0 + 1);
  for (int64_t kt = kt0; kt < kt1; ++kt) {
    __syncthreads();                                                   // the previous tile's readers are done
    if (mover) {
#pragma unroll
      for (int u = 0; u < NP; ++u) {
        const int key = key_first + u * KPP;
        if (key < kKeyTile) st16((char*)(sk + key * KR + 8 * c), stage[u]);
      }
    }
    if (threadIdx.x < kKeyTile) sslot[threadIdx.x] = slot;
    __syncthreads();
    if (kt + 1 < kt1) fetch();
    slot = slot_of(kt + 2);
    f32x4_l sacc[RBW][KBW];
#pragma unroll
    for (int i = 0; i < RBW; ++i)
#pragma unroll
      for (int j = 0; j < KBW; ++j) sacc[i][j] = f32x4_l{0.f, 0.f, 0.f, 0.f};
    // key fragments two steps ahead of their use; the barriers to the scheduler keep it from loading them all at once
    constexpr int AHEAD = 2;
    u32x4 kf[AHEAD + 1][KBW];
    u32x4 qs[AHEAD + 1][RBW];                                          // query fragments that wait in LDS
    auto query_frag = [&](int st, int i) { return sqf[((rg * RBW + i) * (KS - KQ) + st - KQ) * 64 + lane]; };
    auto key_frag = [&](int st, int j) { return ld16((const char*)(sk + (16 * (kg * KBW + j) + r16) * KR + 32 * st + 8 * qd)); };
#pragma unroll
    for (int st = 0; st < AHEAD && st < KS; ++st)
#pragma unroll
      for (int j = 0; j < KBW; ++j) kf[st][j] = key_frag(st, j);
#pragma unroll
    for (int st = 0; st < KS; ++st) {
      if (st + AHEAD < KS) {
#pragma unroll
        for (int j = 0; j < KBW; ++j) kf[(st + AHEAD) % (AHEAD + 1)][j] = key_frag(st + AHEAD, j);
        if (st + AHEAD >= KQ)
#pragma unroll
          for (int i = 0; i < RBW; ++i) qs[(st + AHEAD) % (AHEAD + 1)][i] = query_frag(st + AHEAD, i);
      }
#pragma unroll
      for (int i = 0; i < RBW; ++i) {
        const u32x4 q = st < KQ ? qf[i][st < KQ ? st : 0] : qs[st % (AHEAD + 1)][i];
#pragma unroll
        for (int j = 0; j < KBW; ++j) sacc[i][j] = mfma_l<Tag>(kf[st % (AHEAD + 1)][j], q, sacc[i][j]);
      }
      __builtin_amdgcn_sched_barrier(0);
    }
    float mx[RBW];
    int edge[RBW];                                                     // the last key of this tile the query may see
#pragma unroll
    for (int i = 0; i < RBW; ++i) {
      const int64_t left = qpos[i] - kt * kKeyTile;
      edge[i] = left < 0 ? -1 : (left > kKeyTile ? kKeyTile : (int)left);
      mx[i] = -INFINITY;
#pragma unroll
      for (int j = 0; j < KBW; ++j)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const float v = 16 * (kg * KBW + j) + 4 * qd + r <= edge[i] ? sacc[i][j][r] * scale2 : -INFINITY;
          sacc[i][j][r] = v;
          mx[i] = fmaxf(mx[i], v);
        }
      mx[i] = fmaxf(mx[i], __shfl_xor(mx[i], 16, 64));
      mx[i] = fmaxf(mx[i], __shfl_xor(mx[i], 32, 64));
      if (qd == 0) smax[(wave * RBW + i) * 16 + r16] = mx[i];
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < RBW; ++i) {
      float m_new = m[i];
#pragma unroll
      for (int w = rg; w < NW; w += GROUPS) m_new = fmaxf(m_new, smax[(w * RBW + i) * 16 + r16]);
      // the reference of the exponentials moves only when the maximum has left it by kSlack: sums stay far from overflow, and
      // most tiles need no rescaling
      if (m_new <= m[i] + kSlack) m_new = m[i];
      const float m_safe = m_new == -INFINITY ? 0.f : m_new;           // nothing seen yet: every weight is exp(-inf) = 0
      const float corr = m_new == m[i] ? 1.f : __builtin_amdgcn_exp2f(m[i] - m_safe);
      m[i] = m_new;
      float psum = 0.f;
#pragma unroll
      for (int j = 0; j < KBW; ++j) {
        float p[8], rest[8], back[8];
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          p[r] = __builtin_amdgcn_exp2f(sacc[i][j][r] - m_safe);
          psum += p[r];
          p[4 + r] = 0.f;
        }
        const u32x4 hi = pack16<Tag>(p);
        unpack16<Tag>(hi, back);
#pragma unroll
        for (int r = 0; r < 8; ++r) rest[r] = p[r] - back[r];
        const u32x4 lo = pack16<Tag>(rest);
        u32x2* at = sp_ + ((rg * RBW + i) * 8 + kg * KBW + j) * 64 + lane;
        at[0] = u32x2{hi[0], hi[1]};
        at[4 * 64] = u32x2{lo[0], lo[1]};
      }
      l[i] = l[i] * corr + psum;                                       // this lane's keys only: joined at the end
      if (kg == 0 && qd == 0) scorr[(rg * RBW + i) * 16 + r16] = corr;
    }
    __syncthreads();
    float cr[RB];
#pragma unroll
    for (int i = 0; i < RB; ++i) cr[i] = scorr[i * 16 + r16];
#pragma unroll
    for (int i = 0; i < RB; ++i)
      if (__any(cr[i] != 1.f)) {
#pragma unroll
        for (int d = 0; d < DTW; ++d)
#pragma unroll
          for (int r = 0; r < 4; ++r) oacc[d][i][r] *= cr[i];
      }
#pragma unroll
    for (int hh = 0; hh < 2; ++hh) {
      u32x4 pw[2][RB];                                                 // the weights, their remainders
#pragma unroll
      for (int i = 0; i < RB; ++i)
#pragma unroll
        for (int e = 0; e < 2; ++e) {
          const u32x2* at = sp_ + (i * 8 + 4 * e + 2 * hh) * 64 + lane;
          const u32x2 p0 = at[0], p1 = at[64];
          pw[e][i] = u32x4{p0[0], p0[1], p1[0], p1[1]};
        }
      // lane i of a 16-lane group addresses row 4 qd + (i >> 2), elements 4 (i & 3) .. + 3, and receives column i.  Channels
      // behind C (a wave's last tiles where C < 64 DTW) read the row's other columns; their sums are never stored.
      auto value_frag = [&](int d) {
        const uint16_t* vp = sk + (32 * hh + 4 * qd + (r16 >> 2)) * KR + 16 * (wave * DTW + d) + 4 * (r16 & 3);
        const u32x2 v0 = __builtin_bit_cast(u32x2, __builtin_amdgcn_ds_read_tr16_b64_v4i16(
                                                       (__attribute__((address_space(3))) s16x4_l*)vp));
        const u32x2 v1 = __builtin_bit_cast(u32x2, __builtin_amdgcn_ds_read_tr16_b64_v4i16(
                                                       (__attribute__((address_space(3))) s16x4_l*)(vp + 16 * KR)));
        return u32x4{v0[0], v0[1], v1[0], v1[1]};
      };
      u32x4 vf[2];
      vf[0] = value_frag(0);
#pragma unroll
      for (int d = 0; d < DTW; ++d) {
        if (d + 1 < DTW) vf[(d + 1) & 1] = value_frag(d + 1);
#pragma unroll
        for (int e = 0; e < 2; ++e)
#pragma unroll
          for (int i = 0; i < RB; ++i) oacc[d][i] = mfma_l<Tag>(vf[d & 1], pw[e][i], oacc[d][i]);
        __builtin_amdgcn_sched_barrier(0);
      }
    }
  }
  // denominators: over the lanes of a query, then over the waves that scored its keys
#pragma unroll
  for (int i = 0; i < RBW; ++i) {
    l[i] += __shfl_xor(l[i], 16, 64);
    l[i] += __shfl_xor(l[i], 32, 64);
    if (qd == 0) ssum[(wave * RBW + i) * 16 + r16] = l[i];
  }
  __syncthreads();
  float inv[RB];
#pragma unroll
  for (int i = 0; i < RB; ++i) {
    float den = 0.f;
#pragma unroll
    for (int w = i / RBW; w < NW; w += GROUPS) den += ssum[(w * RBW + i % RBW) * 16 + r16];
    inv[i] = den;
  }
  if (a.splits > 1 && kg == 0 && qd == 0) {
    float* ml = a.part + (int64_t)a.splits * a.T * a.H * a.C;
#pragma unroll
    for (int i = 0; i < RBW; ++i) {
      const int64_t r = row0 + 16 * (rg * RBW + i) + r16;
      if (r < rows) {
        float* at = ml + ((int64_t)blockIdx.y * a.T * a.H + start * a.H + r) * 2;
        at[0] = m[i];
        float den = inv[i];
        const float other = inv[RB - RBW + i];
        if (rg > 0) den = other;
        at[1] = den;
      }
    }
  }
  if (a.splits > 1 && kt0 >= kt1) return;                              // no keys: the merge skips this share
#pragma unroll
  for (int i = 0; i < RB; ++i) {
    const int64_t r = row0 + 16 * i + r16;
    if (r >= rows) continue;
    const int64_t t = start + r / a.H, h = r % a.H;
    const float sc = a.splits > 1 ? 1.f : 1.f / inv[i];
#pragma unroll
    for (int d = 0; d < DTW; ++d) {
      const int ch = 16 * (wave * DTW + d) + 4 * qd;
      if (ch >= a.C) continue;
      float f[8] = {oacc[d][i][0] * sc, oacc[d][i][1] * sc, oacc[d][i][2] * sc, oacc[d][i][3] * sc, 0.f, 0.f, 0.f, 0.f};
      if (a.splits > 1) {
        st16(a.part + ((int64_t)blockIdx.y * a.T * a.H + start * a.H + r) * a.C + ch, pack16<f32_tag>(f));
      } else {
        const u32x4 pk = pack16<Tag>(f);
        *(u32x2*)((char*)a.out + (t * a.lat_token_stride + h * a.lat_head_stride + ch) * 2) = u32x2{pk[0], pk[1]};
      }
    }
  }
}

// one workgroup per row: the shares' sums joined in the order of the keys
template <typename Tag>
__global__ void __launch_bounds__(128) latent_merge_kernel(LatentArgs a) {
  typedef Elem<Tag> E;
  const int64_t r = blockIdx.x, n = a.T * a.H, t = r / a.H, h = r % a.H;
  const float* ml = a.part + (int64_t)a.splits * n * a.C;
  __shared__ float weight[kMaxSplits];
  __shared__ float total;
  __shared__ int last;
  if (threadIdx.x < 64) {                            // a wave: lane s holds share s
    float m = -INFINITY, l = 0.f;
    if ((int)threadIdx.x < a.splits) {
      m = ml[((int64_t)threadIdx.x * n + r) * 2];
      l = ml[((int64_t)threadIdx.x * n + r) * 2 + 1];
    }
    float M = m;
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) M = fmaxf(M, __shfl_xor(M, off, 64));        // (a row has seen itself: M is finite)
    const float w = exp2f(m - M), den = wave_sum(w * l);
    weight[threadIdx.x] = w;
    // shares are dealt from the first key on: all shares up to the last one that saw a key have written a sum
    const unsigned long long seen = __ballot(w > 0.f);
    if (threadIdx.x == 0) {
      total = den;
      last = 63 - __clzll(seen);
    }
  }
  __syncthreads();
  const float inv = 1.f / total;
  for (int c = 4 * threadIdx.x; c < a.C; c += 512) {
    float acc[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
#pragma unroll 8
    for (int s = 0; s <= last; ++s) {
      float f[4];
      unpack16<f32_tag>(ld16(a.part + ((int64_t)s * n + r) * a.C + c), f);
#pragma unroll
      for (int e = 0; e < 4; ++e) acc[e] += weight[s] * f[e];
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) acc[e] *= inv;
    const u32x4 pk = pack16<Tag>(acc);
    *(u32x2*)((char*)a.out + (t * a.lat_token_stride + h * a.lat_head_stride + c) * 2) = u32x2{pk[0], pk[1]};
  }
}

template <typename Tag, int KS, int DT, int RB, int NW>
static int launch_latent_mfma(const LatentArgs& a, const SeqBatch& s, hipStream_t st) {
  constexpr size_t lds = latent_lds<KS, RB, NW>();
  constexpr int DTW = DT / NW;
  if (lds > 64 * 1024) {         // the limit is the device's: raised once per device of the process
    static PerDevice<int> raised;
    int ok = 0;
    raised.get(ok, [&](int) {
      return hipFuncSetAttribute((const void*)latent_mfma_kernel<Tag, KS, DTW, RB, NW>, hipFuncAttributeMaxDynamicSharedMemorySize,
                                 (int)lds) == hipSuccess ? 1 : 0;
    });
    if (!ok) return SP_ERR_LAUNCH;
  }
  const int64_t blocks = s.extend_seq_lens ? (a.T * a.H + 16 * RB - 1) / (16 * RB) + s.B
                                           : (int64_t)s.B * ((a.H + 16 * RB - 1) / (16 * RB));
  latent_mfma_kernel<Tag, KS, DTW, RB, NW><<<dim3((unsigned)blocks, (unsigned)a.splits), 64 * NW, lds, st>>>(a, s);
  SP_LAUNCH_CHECK();
  if (a.splits > 1) {
    latent_merge_kernel<Tag><<<dim3((unsigned)(a.T * a.H)), 128, 0, st>>>(a);
    SP_LAUNCH_CHECK();
  }
  return SP_OK;
}
template <typename Tag, int KS, int DT>
static int launch_latent_rows(const LatentArgs& a, const SeqBatch& s, hipStream_t st) {
  const int64_t rows = s.extend_seq_lens ? 64 : a.H;                   // rows a request brings in a decode step
  if (rows <= 16) return launch_latent_mfma<Tag, KS, DT, 1, 4>(a, s, st);
  if (rows <= 32) return launch_latent_mfma<Tag, KS, DT, 2, 4>(a, s, st);
  return launch_latent_mfma<Tag, KS, DT, 4, (KS > 5 ? 8 : 4)>(a, s, st);      // (narrow rows: more workgroups per CU instead)
}
template <typename Tag>
static int launch_latent(const LatentArgs& a, const SeqBatch& s, hipStream_t st) {
  if (a.C + a.R <= 160 && a.C <= 128) return launch_latent_rows<Tag, 5, 8>(a, s, st);
  if (a.C + a.R <= 320 && a.C <= 256) return launch_latent_rows<Tag, 10, 16>(a, s, st);
  if (a.C + a.R <= 576 && a.C <= 512) return launch_latent_rows<Tag, 18, 32>(a, s, st);
  return SP_ERR_UNSUPPORTED;
}

// ---- out[t, h, n] = sum_k w[h, n, k] x[t, h, k]  (times sigmoid(gate[t, h N + n])) ---------------------------------------
// acc[j][r] of a wave's 16 tokens = out[t + r16][n + 32 (j / 2) + 8 qd + 4 (j % 2) + r]: the output tiles come in pairs, to which
// the rows of w are dealt so that a lane ends with 8 neighbouring outputs of its token (one 16-byte store).  N is a multiple of 4
template <typename Tag, int NT>
__device__ __forceinline__ void head_linear_store(const f32x4_l (&acc)[NT], void* out, int64_t out_stride, int64_t out_head,
                                                  const void* gate, int64_t gate_stride, int64_t t, int n0, int64_t h, int N,
                                                  int qd) {
  const bool whole = N % 8 == 0 && out_stride % 8 == 0 && out_head % 8 == 0 && ((uintptr_t)out & 15) == 0;
  u32x2 half = {0u, 0u};
#pragma unroll
  for (int j = 0; j < NT; ++j) {
    const int n = n0 + (NT % 2 == 0 ? 32 * (j >> 1) + 8 * qd + 4 * (j & 1) : 16 * j + 4 * qd);
    if (n < N) {
      float f[8] = {acc[j][0], acc[j][1], acc[j][2], acc[j][3], 0.f, 0.f, 0.f, 0.f};
      if (gate) {
        float g[8];
        const u32x2 g2 = *(const u32x2*)((const char*)gate + (t * gate_stride + h * N + n) * 2);
        unpack16<Tag>(u32x4{g2[0], g2[1], 0u, 0u}, g);
#pragma unroll
        for (int e = 0; e < 4; ++e) f[e] /= 1.f + expf(-g[e]);
      }
      const u32x4 pk = pack16<Tag>(f);
      char* to = (char*)out + (t * out_stride + h * out_head + n) * 2;
      if (NT % 2 == 0 && whole) {
        if (j % 2 == 0) half = u32x2{pk[0], pk[1]};
        else st16(to - 8, u32x4{half[0], half[1], pk[0], pk[1]});
      } else {
        *(u32x2*)to = u32x2{pk[0], pk[1]};
      }
    }
  }
}

// Few tokens (16-bit): a wave per 16 tokens x 16 outputs of a head, operands straight from memory.
template <typename Tag>
__global__ void __launch_bounds__(256)
head_linear_rows_kernel(void* out, int64_t out_stride, int64_t out_head, const void* x, int64_t x_stride, int64_t x_head,
                        const void* w, const void* gate, int64_t gate_stride, int64_t T, int N, int K) {
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, r16 = lane & 15, qd = lane >> 4;
  const int64_t h = blockIdx.z, t0 = (int64_t)blockIdx.x * 16;
  const int n0 = (blockIdx.y * 4 + wave) * 16;
  if (n0 >= N) return;                                                 // (no workgroup barrier below)
  const int64_t t = t0 + r16 < T ? t0 + r16 : T - 1;
  const int n = n0 + r16 < N ? n0 + r16 : N - 1;
  const char* xp = (const char*)x + (t * x_stride + h * x_head + 8 * qd) * 2;
  const char* wp = (const char*)w + ((h * N + n) * (int64_t)K + 8 * qd) * 2;
  f32x4_l acc[1] = {f32x4_l{0.f, 0.f, 0.f, 0.f}};
  const int whole_k = K / 32 * 32;
#pragma unroll 4
  for (int k = 0; k < whole_k; k += 32) acc[0] = mfma_l<Tag>(ld16(wp + 2 * k), ld16(xp + 2 * k), acc[0]);
  if (whole_k < K) {                                                   // K is a multiple of 8: the lanes behind it bring zeros
    const bool on = whole_k + 8 * qd < K;
    const u32x4 zero = {0u, 0u, 0u, 0u};
    acc[0] = mfma_l<Tag>(on ? ld16(wp + 2 * whole_k) : zero, on ? ld16(xp + 2 * whole_k) : zero, acc[0]);
  }
  if (t0 + r16 < T) head_linear_store<Tag, 1>(acc, out, out_stride, out_head, gate, gate_stride, t0 + r16, n0, h, N, qd);
}

// Many tokens (16-bit): 128 tokens x TN outputs of a head per workgroup, both operands staged in LDS 64 columns at a time (whole
// 128-byte lines per 8 lanes; an operand fragment taken straight from memory touches 16 lines per 16 lanes), the next columns in
// flight during the products.  TN = 128: the 4 waves form 64 x 64 each; TN = 64: 32 x 64.
constexpr int kHeadRow = 72;                                           // 64 columns + 16 bytes that spread the rows over the banks
template <typename Tag, int TN>
__global__ void __launch_bounds__(256)
head_linear_tile_kernel(void* out, int64_t out_stride, int64_t out_head, const void* x, int64_t x_stride, int64_t x_head,
                        const void* w, const void* gate, int64_t gate_stride, int64_t T, int N, int K) {
  constexpr int WN = TN / 64, WT = 4 / WN, TT = 8 / WT, NT = 4, XP = 4, WP = TN / 32;
  __shared__ __attribute__((aligned(16))) uint16_t sx[128 * kHeadRow], sw[TN * kHeadRow];
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, r16 = lane & 15, qd = lane >> 4;
  const int64_t h = blockIdx.z, t0 = (int64_t)blockIdx.x * 128;
  const int n0 = blockIdx.y * TN, row = threadIdx.x >> 3, col = 8 * (threadIdx.x & 7);
  const char *xp[XP], *wp[WP];
  int xl[XP], wl[WP];                                                  // where a piece lies in LDS
#pragma unroll
  for (int u = 0; u < XP; ++u) {
    const int r = row + 32 * u;
    xp[u] = (const char*)x + ((t0 + r < T ? t0 + r : T - 1) * x_stride + h * x_head) * 2;
    xl[u] = r * kHeadRow + col;
  }
#pragma unroll
  for (int u = 0; u < WP; ++u) {
    const int r = row + 32 * u, m = r & 63;                            // output r of the tile -> row 16 j + r16 of its group of 64
    wp[u] = (const char*)w + (h * N + (n0 + r < N ? n0 + r : N - 1)) * (int64_t)K * 2;
    wl[u] = ((r & 64) + 16 * (2 * (m >> 5) + ((m >> 2) & 1)) + 4 * ((m >> 3) & 3) + (m & 3)) * kHeadRow + col;
  }
  u32x4 fx[XP], fw[WP];
  auto fetch = [&](int k0) {                                           // columns behind K: the last ones again, as zeros
    const int k = k0 + col, kc = 2 * (k < K ? k : K - 8);
    const uint32_t keep = k < K ? 0xffffffffu : 0u;
#pragma unroll
    for (int u = 0; u < XP; ++u) fx[u] = ld16(xp[u] + kc);
#pragma unroll
    for (int u = 0; u < WP; ++u) fw[u] = ld16(wp[u] + kc);
    if (k0 + 64 > K) {
#pragma unroll
      for (int u = 0; u < XP; ++u) fx[u] &= keep;
#pragma unroll
      for (int u = 0; u < WP; ++u) fw[u] &= keep;
    }
  };
  f32x4_l acc[TT][NT];
#pragma unroll
  for (int i = 0; i < TT; ++i)
#pragma unroll
    for (int j = 0; j < NT; ++j) acc[i][j] = f32x4_l{0.f, 0.f, 0.f, 0.f};
  const int tw = (wave / WN) * 16 * TT, nw = (wave % WN) * 64;         // this wave's corner of the tile
  fetch(0);
  for (int k0 = 0; k0 < K; k0 += 64) {
    __syncthreads();                                                   // the previous columns' readers are done
#pragma unroll
    for (int u = 0; u < XP; ++u) st16(sx + xl[u], fx[u]);
#pragma unroll
    for (int u = 0; u < WP; ++u) st16(sw + wl[u], fw[u]);
    __syncthreads();
    if (k0 + 64 < K) fetch(k0 + 64);
#pragma unroll
    for (int st = 0; st < 2; ++st) {
      u32x4 xf[TT], wf[NT];
#pragma unroll
      for (int i = 0; i < TT; ++i) xf[i] = ld16(sx + (tw + 16 * i + r16) * kHeadRow + 32 * st + 8 * qd);
#pragma unroll
      for (int j = 0; j < NT; ++j) wf[j] = ld16(sw + (nw + 16 * j + r16) * kHeadRow + 32 * st + 8 * qd);
#pragma unroll
      for (int i = 0; i < TT; ++i)
#pragma unroll
        for (int j = 0; j < NT; ++j) acc[i][j] = mfma_l<Tag>(wf[j], xf[i], acc[i][j]);
    }
  }
#pragma unroll
  for (int i = 0; i < TT; ++i) {
    const int64_t t = t0 + tw + 16 * i + r16;
    if (t < T) head_linear_store<Tag, NT>(acc[i], out, out_stride, out_head, gate, gate_stride, t, n0 + nw, h, N, qd);
  }
}

// any type, size and alignment: one workgroup per (token, head), the token's row in LDS, a thread per output
template <typename Tag>
__global__ void __launch_bounds__(kBlock)
head_linear_kernel(void* out, int64_t out_stride, int64_t out_head, const void* x, int64_t x_stride, int64_t x_head,
                   const void* w, const void* gate, int64_t gate_stride, int N, int K) {
  typedef Elem<Tag> E;
  extern __shared__ float smem[];
  const int64_t t = blockIdx.x, h = blockIdx.y;
  for (int k = threadIdx.x; k < K; k += blockDim.x) smem[k] = E::load(x, t * x_stride + h * x_head + k);
  __syncthreads();
  for (int n = threadIdx.x; n < N; n += blockDim.x) {
    const int64_t row = (h * N + n) * (int64_t)K;
    float acc = 0.f;
    for (int k = 0; k < K; ++k) acc += smem[k] * E::load(w, row + k);
    if (gate) acc /= 1.f + expf(-E::load(gate, t * gate_stride + h * N + n));
    E::store(out, t * out_stride + h * out_head + n, acc);
  }
}

}  // namespace
}  // namespace sp

using namespace sp;

extern "C" int sp_rotary_interleaved(void* x, const int64_t* positions, const float* freq, float mag, int64_t num_tokens,
                                     int heads, int rot_dim, int64_t token_stride, int64_t head_stride, int offset,
                                     int dtype, void* stream) {
  SP_CHECK_ARG(num_tokens >= 0 && heads > 0 && rot_dim >= 0 && rot_dim % 2 == 0 && offset >= 0);
  if (num_tokens == 0 || rot_dim == 0) return SP_OK;
  SP_CHECK_ARG(x && positions && freq);
  SP_DISPATCH_DTYPE(dtype, (rotary_interleaved_kernel<Tag><<<dim3((unsigned)num_tokens), kBlock, 0, (hipStream_t)stream>>>(
                               x, positions, freq, mag, heads, rot_dim, token_stride, head_stride, offset)));
  SP_LAUNCH_CHECK();
  return SP_OK;
}

extern "C" int sp_latent_kv_store(void* pool, int64_t pool_stride, const void* dkv, int64_t dkv_stride,
                                  const float* norm_w, void* q, int64_t q_stride, int64_t q_head_stride, int q_offset,
                                  int heads, const int64_t* positions, const float* freq, float mag, const int64_t* loc,
                                  int64_t num_tokens, int rank, int rot_dim, int rot_dims, float eps, int dtype, void* stream) {
  SP_CHECK_ARG(num_tokens >= 0 && rank > 0 && rot_dim >= 0 && rot_dims >= 0 && rot_dims <= rot_dim && rot_dims % 2 == 0);
  if (num_tokens == 0) return SP_OK;
  SP_CHECK_ARG((pool || q) && positions && (freq || rot_dims == 0));
  SP_CHECK_ARG(!pool || (dkv && norm_w && loc && pool_stride >= rank + rot_dim && dkv_stride >= rank + rot_dim));
  SP_CHECK_ARG(!q || (heads > 0 && q_offset >= 0 && q_head_stride >= q_offset + rot_dims));
  if (rot_dims > kMaxRot) return SP_ERR_UNSUPPORTED;
  SP_DISPATCH_DTYPE(dtype, (latent_kv_store_kernel<Tag><<<dim3((unsigned)num_tokens), kBlock, 0, (hipStream_t)stream>>>(
                               pool, pool_stride, dkv, dkv_stride, norm_w, q, q_stride, q_head_stride, q_offset, heads, positions,
                               freq, mag, loc, rank, rot_dim, rot_dims, eps)));
  SP_LAUNCH_CHECK();
  return SP_OK;
}

extern "C" int sp_latent_attention(void* out, const void* q_lat, int64_t lat_token_stride, int64_t lat_head_stride,
                                   const void* q_rot, const void* pool, int64_t pool_stride, const int32_t* req_to_token,
                                   int64_t table_stride, int64_t num_tokens, int heads, int rank, int rot_dim,
                                   int64_t qrot_token_stride, int64_t qrot_head_stride, float scale, int matrix, int splits,
                                   float* workspace, int64_t workspace_floats, SP_SEQ_PARAMS, int dtype, void* stream) {
  SP_CHECK_ARG(num_tokens >= 0 && heads > 0 && rank > 0 && rot_dim >= 0);
  if (num_tokens == 0) return SP_OK;
  SP_CHECK_ARG(out && q_lat && pool && req_to_token && req_pool_indices && seq_lens && (q_rot || rot_dim == 0));
  SP_CHECK_ARG(!extend_seq_lens || (extend_prefix_lens && extend_start_loc && token_req));
  SP_CHECK_ARG(extend_seq_lens || num_tokens == batch_size);
  SP_CHECK_ARG(pool_stride >= rank + rot_dim && lat_token_stride >= rank && lat_head_stride >= rank);
  SEQ_BATCH(s);
  // 16-bit rows of whole 16-byte pieces, widths the tile shapes cover: the matrix cores; anything else: the vector kernel
  const bool al16 = (((uintptr_t)q_lat | (uintptr_t)q_rot | (uintptr_t)pool | (uintptr_t)workspace) & 15) == 0 &&
                    ((uintptr_t)out & 7) == 0;
  if (matrix && (dtype == SP_BF16 || dtype == SP_F16) && rank % 8 == 0 && rot_dim % 8 == 0 && rank <= 512 &&
      rank + rot_dim <= 576 && al16 && lat_token_stride % 8 == 0 && lat_head_stride % 8 == 0 && qrot_token_stride % 8 == 0 &&
      qrot_head_stride % 8 == 0 && pool_stride % 8 == 0) {
    if (splits < 1) splits = 1;
    SP_CHECK_ARG(splits == 1 || (workspace && splits <= kMaxSplits));
    if (splits > 1 && workspace_floats < (int64_t)splits * num_tokens * heads * (rank + 2)) return SP_ERR_WORKSPACE;
    const LatentArgs a{out, q_lat, q_rot, pool, req_to_token, workspace, lat_token_stride, lat_head_stride, qrot_token_stride,
                       qrot_head_stride, pool_stride, table_stride, num_tokens, heads, rank, rot_dim, splits, scale};
    return dtype == SP_BF16 ? launch_latent<bf16_tag>(a, s, (hipStream_t)stream)
                            : launch_latent<f16_tag>(a, s, (hipStream_t)stream);
  }
  if (rank > 64 * kMaxPerLane) return SP_ERR_UNSUPPORTED;
  const size_t lds = 4 * (size_t)(rank + rot_dim + 64) * sizeof(float);
  if (lds > 64 * 1024) return SP_ERR_UNSUPPORTED;
  const dim3 grid((unsigned)num_tokens, (unsigned)((heads + 3) / 4));
  SP_DISPATCH_DTYPE(dtype, (latent_attention_kernel<Tag><<<grid, 256, lds, (hipStream_t)stream>>>(
                               out, q_lat, lat_token_stride, lat_head_stride, q_rot, pool, pool_stride, req_to_token, table_stride,
                               s, num_tokens, heads, rank, rot_dim, qrot_token_stride, qrot_head_stride, scale)));
  SP_LAUNCH_CHECK();
  return SP_OK;
}

extern "C" int sp_head_linear(void* out, int64_t out_stride, int64_t out_head_stride, const void* x, int64_t x_stride,
                              int64_t x_head_stride, const void* w, const void* gate, int64_t gate_stride,
                              int64_t num_tokens, int heads, int n, int k, int dtype, void* stream) {
  SP_CHECK_ARG(num_tokens >= 0 && heads > 0 && n > 0 && k > 0);
  if (num_tokens == 0) return SP_OK;
  SP_CHECK_ARG(out && x && w && x_head_stride >= k && out_head_stride >= n && heads <= 65535);
  SP_CHECK_ARG(x_stride >= (heads - 1) * x_head_stride + k && out_stride >= (heads - 1) * out_head_stride + n);
  SP_CHECK_ARG(!gate || gate_stride >= (int64_t)heads * n);
  const bool al = (((uintptr_t)x | (uintptr_t)w) & 15) == 0 && (((uintptr_t)out | (uintptr_t)gate) & 7) == 0 &&
                  x_stride % 8 == 0 && x_head_stride % 8 == 0 && k % 8 == 0 && n % 4 == 0 && out_stride % 4 == 0 &&
                  out_head_stride % 4 == 0 && (!gate || gate_stride % 4 == 0);
  hipStream_t st = (hipStream_t)stream;
  if (al && (dtype == SP_BF16 || dtype == SP_F16)) {
#define SP_HL(KERNEL, TILE_T, TILE_N)                                                                                   \
  KERNEL<<<dim3((unsigned)((num_tokens + TILE_T - 1) / TILE_T), (unsigned)((n + TILE_N - 1) / TILE_N), (unsigned)heads), 256, 0, \
           st>>>(out, out_stride, out_head_stride, x, x_stride, x_head_stride, w, gate, gate_stride, num_tokens, n, k)
#define SP_HL_TYPES(TILE_T, TILE_N, NAME, ...)                                     \
  do {                                                                             \
    if (dtype == SP_BF16) SP_HL((NAME<bf16_tag __VA_ARGS__>), TILE_T, TILE_N);     \
    else SP_HL((NAME<f16_tag __VA_ARGS__>), TILE_T, TILE_N);                       \
  } while (0)
    if (num_tokens <= 64) SP_HL_TYPES(16, 64, head_linear_rows_kernel);
    else if (n > 64) SP_HL_TYPES(128, 128, head_linear_tile_kernel, , 128);
    else SP_HL_TYPES(128, 64, head_linear_tile_kernel, , 64);
#undef SP_HL_TYPES
#undef SP_HL
    SP_LAUNCH_CHECK();
    return SP_OK;
  }
  const size_t lds = (size_t)k * sizeof(float);
  if (lds > 64 * 1024) return SP_ERR_UNSUPPORTED;
  SP_DISPATCH_DTYPE(dtype, (head_linear_kernel<Tag><<<dim3((unsigned)num_tokens, (unsigned)heads), kBlock, lds, st>>>(
                               out, out_stride, out_head_stride, x, x_stride, x_head_stride, w, gate, gate_stride, n, k)));
  SP_LAUNCH_CHECK();
  return SP_OK;
}
