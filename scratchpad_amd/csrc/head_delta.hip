// Head-gated delta rule: a per-head matrix state S [D, Dv] that decays by ONE factor per token and head and is corrected
// along the unit key.  Per value head h (its query/key head is h / (H / G)), all of the recurrence in fp32:
//   qn = q / sqrt(|q|^2 + 1e-6) * D^(-1/2)        kn = k / sqrt(|k|^2 + 1e-6)
//   beta = sigmoid(bpre)                          g = exp(-exp(A_log) softplus(apre + dt_bias))
//   S  = g S;   u = beta (v - S^T kn);   S = S + kn u^T;   o = S^T qn       (the read-out sees the token's own write)
//   out = o / rms_head(o) * norm_w * silu(gate)   (norm_w [Dv] shared by the heads)
// Both gates are formed from their fp32 pre-activations where they are used.
//
// A workgroup owns a range of a head's value channels (columns of S) for one request and walks the request's tokens of this
// step in order from the state the previous step left in the pool (zeros at a sequence's first token).  SP neighbouring lanes
// share 4 columns: a lane keeps D / SP rows of each in registers, so one value of q and k read from LDS serves four columns -
// the traffic between LDS and registers, not the arithmetic, is what bounds a column per lane.  A token costs ONE sweep: the
// update, the read-out and, on the state just completed, the next token's S^T kn (its decay is a factor of the whole sum),
// then sums over the SP lanes by register moves; no workgroup barrier inside a pass of kChunk tokens.
// With one range per head the norm and the gate are the pass's epilogue; where a step brings long portions of few requests,
// several workgroups share a head and hand fp32 read-outs to head_norm_gate_kernel.  Prompt portions and single decoded
// tokens take the same path, and the order of every sum depends on the head's sizes only.
#include "seq_batch.h"

namespace sp {
namespace {

__device__ __forceinline__ float softplus_hd(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }

constexpr int kCols = 4;                                          // columns of S per lane
constexpr int hd_chunk(int KP) { return KP > 128 ? 8 : 16; }      // tokens staged in LDS per pass
constexpr int hd_lanes(int KP) { return KP >= 64 ? 16 : KP / 4; } // lanes that share a column
constexpr int kHdMaxV = 256;                                      // value channels per head

struct HeadDelta {
  void* out;
  float* raw;                 // several workgroups per head: o as read out, fp32 [T, H * Dv]
  const void *q, *k, *v, *gate;
  const float *pre, *dt_bias, *A_log, *norm_w;      // pre [T, >= 2 H]: bpre of every head, then apre of every head
  float* state;
  int64_t out_stride, q_stride, k_stride, v_stride, gate_stride, pre_stride, state_stride;
  int H, G, K, Dv, cols;      // cols: columns per workgroup
  float eps;
};

// sum over aligned groups of N lanes, N a power of two up to a wave
template <int N>
__device__ __forceinline__ float group_sum(float v) {
  v = lanes_sum<(N < 16 ? N : 16)>(v);
  if constexpr (N >= 32) v += __shfl_xor(v, 16, 64);
  if constexpr (N >= 64) v += __shfl_xor(v, 32, 64);
  return v;
}

template <typename Tag, int KP, bool VEC, int MAXT>
__global__ void __launch_bounds__(MAXT)
head_delta_kernel(HeadDelta a, SeqBatch s) {
  typedef Elem<Tag> E;
  constexpr int kChunk = hd_chunk(KP), SP = hd_lanes(KP), DS = KP / SP, V = E::kVec;
  static_assert(DS % 4 == 0, "a lane's rows are read four at a time");
  extern __shared__ __attribute__((aligned(16))) float smem[];
  const int cols = a.cols, K = a.K, H = a.H, Dv = a.Dv;
  float* sq = smem;                                  // [kChunk][KP]
  float* sk = sq + kChunk * KP;                      // [kChunk + 1][KP]
  float* sv = sk + (kChunk + 1) * KP;                // [kChunk][cols]
  float* so = sv + kChunk * cols;                    // [kChunk][cols]
  float* sg = so + kChunk * cols;                    // [kChunk] decay
  float* sbeta = sg + kChunk;                        // [kChunk]
  float* sinv = sbeta + kChunk;                      // [kChunk]
  const int b = blockIdx.x, h = blockIdx.y, j = threadIdx.x, NT = blockDim.x;
  const int wave = j >> 6, lane = j & 63, waves = NT >> 6;
  const int col0 = blockIdx.z * cols;                // this workgroup's columns of the head: col0 .. col0 + ncols
  const int ncols = Dv - col0 < cols ? Dv - col0 : cols;
  const int cg = j / SP, part = j % SP, c0 = cg * kCols;
  int64_t start, len, prefix;
  seq_span(s, b, start, len, prefix);
  if (len <= 0) return;
  const int gh = h / (H / a.G);
  float* st = a.state + load_idx(s.req_pool_indices, b, s.idx64) * a.state_stride + (int64_t)h * K * Dv + col0;
  const bool held = prefix > 0;
  const int64_t qc = (int64_t)gh * K, vc = (int64_t)h * Dv + col0;
  const float qscale = 1.f / sqrtf((float)K), rate = expf(a.A_log[h]), bias = a.dt_bias[h];
  // rows of whole 16-byte pieces: a lane moves its 4 columns of a row at once
  const bool quad = Dv % 4 == 0 && a.state_stride % 4 == 0 && ((uintptr_t)a.state & 15) == 0;
  // lane `part` owns the rows 4 part + e + 4 SP jj of its columns: the lanes of a column read one contiguous stretch of LDS
  float S[kCols][DS];
#pragma unroll
  for (int ii = 0; ii < DS; ++ii) {
    const int i = 4 * part + (ii & 3) + 4 * SP * (ii >> 2);
    if (quad) {
      float4 x = {0.f, 0.f, 0.f, 0.f};
      if (held && i < K && c0 < ncols) x = *reinterpret_cast<const float4*>(st + (int64_t)i * Dv + c0);
      S[0][ii] = x.x, S[1][ii] = x.y, S[2][ii] = x.z, S[3][ii] = x.w;
    } else {
#pragma unroll
      for (int c = 0; c < kCols; ++c) S[c][ii] = (held && i < K && c0 + c < ncols) ? st[(int64_t)i * Dv + c0 + c] : 0.f;
    }
  }
  // staging in 16-byte pieces: QP pieces (lanes) per row of q and k, vp per row of this workgroup's values
  constexpr int kAhead = 2, QP = KP / V;
  const int vp = cols / V;
  u32x4 fq[kAhead], fk[kAhead], fv[kAhead];
  float fb = 0.f, fa = 0.f;
  auto get_qk = [&](int e, int64_t t0, int n, u32x4& rq, u32x4& rk) {
    const int tt = e / QP, i = (e % QP) * V;
    const int64_t row = start + t0 + tt;
    rq = rk = u32x4{0u, 0u, 0u, 0u};
    if (tt < n && i < K) {
      rq = ld16((const char*)a.q + (row * a.q_stride + qc + i) * E::kBytes);
      rk = ld16((const char*)a.k + (row * a.k_stride + qc + i) * E::kBytes);
    }
  };
  auto get_v = [&](int e, int64_t t0, int n, u32x4& rv) {
    const int tt = e / vp, i = (e % vp) * V;
    rv = u32x4{0u, 0u, 0u, 0u};
    if (tt < n && i < ncols) rv = ld16((const char*)a.v + ((start + t0 + tt) * a.v_stride + vc + i) * E::kBytes);
  };
  auto get_gates = [&](int64_t t0, int n, float& b_, float& a_) {
    if (j < n) {
      const float* pre = a.pre + (start + t0 + j) * a.pre_stride;
      b_ = pre[h];
      a_ = pre[H + h];
    }
  };
  auto put_qk = [&](int e, int n, const u32x4& rq, const u32x4& rk) {
    const int tt = e / QP;
    if (tt >= n) return;                             // (all lanes of a row or none)
    float q_[V], k_[V], q2 = 0.f, k2 = 0.f;
    unpack16<Tag>(rq, q_);
    unpack16<Tag>(rk, k_);
#pragma unroll
    for (int x = 0; x < V; ++x) {
      q2 += q_[x] * q_[x];
      k2 += k_[x] * k_[x];
    }
    const float iq = qscale * rsqrtf(group_sum<QP>(q2) + 1e-6f), ik = rsqrtf(group_sum<QP>(k2) + 1e-6f);
#pragma unroll
    for (int x = 0; x < V; ++x) {
      q_[x] *= iq;
      k_[x] *= ik;
    }
#pragma unroll
    for (int x = 0; x < V; x += 4) {
      st16(sq + e * V + x, pack16<f32_tag>(q_ + x));
      st16(sk + e * V + x, pack16<f32_tag>(k_ + x));
    }
  };
  auto put_v = [&](int e, int n, const u32x4& rv) {
    if (e >= n * vp) return;
    float v_[V];
    unpack16<Tag>(rv, v_);
#pragma unroll
    for (int x = 0; x < V; x += 4) st16(sv + e * V + x, pack16<f32_tag>(v_ + x));
  };
  auto put_gates = [&](float b_, float a_) {
    sbeta[j] = 1.f / (1.f + expf(-b_));
    sg[j] = expf(-rate * softplus_hd(a_ + bias));
  };
  auto fetch = [&](int64_t t0) {
    const int n = (int)(len - t0 < kChunk ? len - t0 : kChunk);
#pragma unroll
    for (int u = 0; u < kAhead; ++u) {
      get_qk(j + u * NT, t0, n, fq[u], fk[u]);
      get_v(j + u * NT, t0, n, fv[u]);
    }
    get_gates(t0, n, fb, fa);
  };
  // which columns of which tokens this thread hands on (several workgroups per head): its column group, every o_step-th token
  const int og = (ncols + kCols - 1) / kCols, o_step = NT / og, o_col = (j % og) * kCols;
  const int o_row = j < og * o_step ? j / og : kChunk;
  if constexpr (VEC) fetch(0);
  for (int64_t t0 = 0; t0 < len; t0 += kChunk) {
    const int n = (int)(len - t0 < kChunk ? len - t0 : kChunk);
    __syncthreads();                                 // the previous pass's readers are done
    if constexpr (VEC) {
      // the pieces fetched during the previous pass's token loop, then (small workgroups) what they did not cover: a row's
      // lanes hold all of it, so its norm is formed on the way
#pragma unroll
      for (int u = 0; u < kAhead; ++u) put_qk(j + u * NT, n, fq[u], fk[u]);
#pragma unroll
      for (int u = 0; u < kAhead; ++u) put_v(j + u * NT, n, fv[u]);
      for (int e = j + kAhead * NT; e < n * QP; e += NT) {
        u32x4 rq, rk;
        get_qk(e, t0, n, rq, rk);
        put_qk(e, n, rq, rk);
      }
      for (int e = j + kAhead * NT; e < n * vp; e += NT) {
        u32x4 rv;
        get_v(e, t0, n, rv);
        put_v(e, n, rv);
      }
      if (j < n) put_gates(fb, fa);
    } else {
      for (int e = j; e < n * KP; e += NT) {
        const int tt = e / KP, i = e % KP;
        const int64_t row = start + t0 + tt;
        sq[e] = i < K ? E::load(a.q, row * a.q_stride + qc + i) : 0.f;
        sk[e] = i < K ? E::load(a.k, row * a.k_stride + qc + i) : 0.f;
      }
      for (int e = j; e < n * cols; e += NT) {
        const int tt = e / cols, i = e % cols;
        sv[e] = i < ncols ? E::load(a.v, (start + t0 + tt) * a.v_stride + vc + i) : 0.f;
      }
      if (j < n) {
        get_gates(t0, n, fb, fa);
        put_gates(fb, fa);
      }
      __syncthreads();
      for (int tt = wave; tt < n; tt += waves) {     // unit query and key of every token of the pass: a wave per token
        float sk2 = 0.f, sq2 = 0.f;
        for (int i = lane; i < K; i += 64) {
          sk2 += sk[tt * KP + i] * sk[tt * KP + i];
          sq2 += sq[tt * KP + i] * sq[tt * KP + i];
        }
        const float ik = 1.f / sqrtf(wave_sum(sk2) + 1e-6f), iq = qscale / sqrtf(wave_sum(sq2) + 1e-6f);
        for (int i = lane; i < K; i += 64) {
          sk[tt * KP + i] *= ik;
          sq[tt * KP + i] *= iq;
        }
      }
    }
    __syncthreads();
    if constexpr (VEC) {
      if (t0 + kChunk < len) fetch(t0 + kChunk);
    }
    float k[DS], proj[kCols];
    {
      float pj[kCols] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ii = 0; ii < DS; ii += 4) {
        const float4 k4 = *reinterpret_cast<const float4*>(sk + 4 * part + SP * ii);
        k[ii] = k4.x, k[ii + 1] = k4.y, k[ii + 2] = k4.z, k[ii + 3] = k4.w;
      }
#pragma unroll
      for (int ii = 0; ii < DS; ++ii)
#pragma unroll
        for (int c = 0; c < kCols; ++c) pj[c] += k[ii] * S[c][ii];
#pragma unroll
      for (int c = 0; c < kCols; ++c) proj[c] = lanes_sum<SP>(pj[c]);
    }
    const bool live = c0 < ncols;
    const int cl = live ? c0 : 0;                    // (lanes behind the last column compute on the first, and store nothing)
    // a token's operands are in registers when its turn comes; the next token's are on their way (behind the pass's last row
    // these reads meet LDS of other arrays, and what they return is never used)
    struct Operands {
      float q[DS], kn[DS];                           // its query, the NEXT token's key
      float4 v;
      float g, beta;
    } cur, nxt;
    auto read = [&](int tt, Operands& o) {
      const float* pq = sq + tt * KP + 4 * part;
      const float* pk = sk + (tt + 1) * KP + 4 * part;
#pragma unroll
      for (int ii = 0; ii < DS; ii += 4) {
        const float4 q4 = *reinterpret_cast<const float4*>(pq + SP * ii), n4 = *reinterpret_cast<const float4*>(pk + SP * ii);
        o.q[ii] = q4.x, o.q[ii + 1] = q4.y, o.q[ii + 2] = q4.z, o.q[ii + 3] = q4.w;
        o.kn[ii] = n4.x, o.kn[ii + 1] = n4.y, o.kn[ii + 2] = n4.z, o.kn[ii + 3] = n4.w;
      }
      o.v = *reinterpret_cast<const float4*>(sv + tt * cols + cl);
      o.g = sg[tt];
      o.beta = sbeta[tt];
    };
    // S with the token that has key kt and operands o; its read-out to LDS, the next token's S^T kn to proj
    auto token = [&](int tt, const float* kt, const Operands& o) {
      const float u[kCols] = {o.beta * (o.v.x - o.g * proj[0]), o.beta * (o.v.y - o.g * proj[1]),
                              o.beta * (o.v.z - o.g * proj[2]), o.beta * (o.v.w - o.g * proj[3])};
      float nm[kCols] = {0.f, 0.f, 0.f, 0.f}, pj[kCols] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int ii = 0; ii < DS; ++ii)
#pragma unroll
        for (int c = 0; c < kCols; ++c) {
          const float x = o.g * S[c][ii] + kt[ii] * u[c];
          S[c][ii] = x;
          nm[c] += x * o.q[ii];
          pj[c] += x * o.kn[ii];
        }
#pragma unroll
      for (int c = 0; c < kCols; ++c) {
        nm[c] = lanes_sum<SP>(nm[c]);
        proj[c] = lanes_sum<SP>(pj[c]);
      }
      if (live && part == 0) *reinterpret_cast<float4*>(so + tt * cols + c0) = float4{nm[0], nm[1], nm[2], nm[3]};
    };
    read(0, cur);
    int tt = 0;
    for (; tt + 2 <= n; tt += 2) {                   // two tokens per round: the operands change names, not registers
      read(tt + 1, nxt);
      token(tt, k, cur);
      float kc[DS];
#pragma unroll
      for (int ii = 0; ii < DS; ++ii) kc[ii] = cur.kn[ii];
      read(tt + 2, cur);
      token(tt + 1, kc, nxt);
#pragma unroll
      for (int ii = 0; ii < DS; ++ii) k[ii] = nxt.kn[ii];
    }
    if (tt < n) token(tt, k, cur);
    __syncthreads();
    if (a.raw) {                                     // the head's other columns are other workgroups': norm and gate follow
      for (int r = o_row; r < n; r += o_step) {
        const float4 x = *reinterpret_cast<const float4*>(so + r * cols + o_col);
        float* to = a.raw + (start + t0 + r) * (int64_t)H * Dv + vc + o_col;
        if (quad) {
          *reinterpret_cast<float4*>(to) = x;
        } else {
          const float xs[kCols] = {x.x, x.y, x.z, x.w};
#pragma unroll
          for (int c = 0; c < kCols; ++c)
            if (o_col + c < ncols) to[c] = xs[c];
        }
      }
      continue;
    }
    for (int tt = wave; tt < n; tt += waves) {
      float ss = 0.f;
      for (int i = lane; i < Dv; i += 64) ss += so[tt * cols + i] * so[tt * cols + i];
      ss = wave_sum(ss);
      if (lane == 0) sinv[tt] = 1.f / sqrtf(ss / (float)Dv + a.eps);
    }
    __syncthreads();
    for (int e = j; e < n * Dv; e += NT) {
      const int tt = e / Dv, i = e % Dv;
      const int64_t row = start + t0 + tt;
      const float z = E::load(a.gate, row * a.gate_stride + vc + i);
      E::store(a.out, row * a.out_stride + vc + i, so[tt * cols + i] * sinv[tt] * a.norm_w[i] * (z / (1.f + expf(-z))));
    }
  }
#pragma unroll
  for (int ii = 0; ii < DS; ++ii) {
    const int i = 4 * part + (ii & 3) + 4 * SP * (ii >> 2);
    if (quad) {
      if (i < K && c0 < ncols) *reinterpret_cast<float4*>(st + (int64_t)i * Dv + c0) = float4{S[0][ii], S[1][ii], S[2][ii], S[3][ii]};
    } else {
#pragma unroll
      for (int c = 0; c < kCols; ++c)
        if (i < K && c0 + c < ncols) st[(int64_t)i * Dv + c0 + c] = S[c][ii];
    }
  }
}

// out[t, h] = raw[t, h] / rms * norm_w * silu(gate[t, h]): a wave per (token, head)
template <typename Tag>
__global__ void __launch_bounds__(kBlock) head_norm_gate_kernel(HeadDelta a, int64_t jobs) {
  typedef Elem<Tag> E;
  const int lane = threadIdx.x & 63, Dv = a.Dv;
  const int64_t job = (int64_t)blockIdx.x * (kBlock / 64) + (threadIdx.x >> 6);
  if (job >= jobs) return;
  const int64_t t = job / a.H, h = job % a.H;
  const float* o = a.raw + job * Dv;
  float f[kHdMaxV / 64], ss = 0.f;
#pragma unroll
  for (int u = 0; u < kHdMaxV / 64; ++u) {
    const int i = lane + 64 * u;
    f[u] = i < Dv ? o[i] : 0.f;
    ss += f[u] * f[u];
  }
  const float inv = 1.f / sqrtf(wave_sum(ss) / (float)Dv + a.eps);
#pragma unroll
  for (int u = 0; u < kHdMaxV / 64; ++u) {
    const int i = lane + 64 * u;
    if (i < Dv) {
      const float z = E::load(a.gate, t * a.gate_stride + h * Dv + i);
      E::store(a.out, t * a.out_stride + h * Dv + i, f[u] * inv * a.norm_w[i] * (z / (1.f + expf(-z))));
    }
  }
}

template <typename Tag, int KP>
static int launch_hd(const HeadDelta& a, const SeqBatch& s, int ranges, bool vec, int64_t T, hipStream_t st) {
  constexpr int SP = hd_lanes(KP), CH = hd_chunk(KP);
  const dim3 grid((unsigned)s.B, (unsigned)a.H, (unsigned)ranges);
  const unsigned threads = (unsigned)(((a.cols + kCols - 1) / kCols * SP + 63) / 64 * 64);
  const size_t lds = ((size_t)(2 * CH + 1) * KP + 2 * CH * a.cols + 3 * CH) * sizeof(float);
  static_assert(((2 * CH + 1) * KP + 2 * CH * kHdMaxV + 3 * CH) * sizeof(float) <= 64 * 1024, "LDS of the widest head");
  if (threads <= 512) {          // (a larger workgroup leaves a lane half the registers)
    if (vec) head_delta_kernel<Tag, KP, true, 512><<<grid, threads, lds, st>>>(a, s);
    else head_delta_kernel<Tag, KP, false, 512><<<grid, threads, lds, st>>>(a, s);
  } else {
    if (vec) head_delta_kernel<Tag, KP, true, 1024><<<grid, threads, lds, st>>>(a, s);
    else head_delta_kernel<Tag, KP, false, 1024><<<grid, threads, lds, st>>>(a, s);
  }
  SP_LAUNCH_CHECK();
  if (a.raw) {
    const int64_t jobs = T * a.H;
    head_norm_gate_kernel<Tag><<<dim3((unsigned)((jobs + kBlock / 64 - 1) / (kBlock / 64))), kBlock, 0, st>>>(a, jobs);
    SP_LAUNCH_CHECK();
  }
  return SP_OK;
}

}  // namespace
}  // namespace sp

using namespace sp;

extern "C" int sp_head_delta_scan(void* out, int64_t out_stride, const void* q, int64_t q_stride, const void* k,
                                  int64_t k_stride, const void* v, int64_t v_stride, const void* gate, int64_t gate_stride,
                                  const float* pre, int64_t pre_stride, const float* dt_bias, const float* A_log,
                                  const float* norm_w, float* state, int64_t state_stride, float* workspace,
                                  int64_t num_tokens, int heads, int kv_heads, int dim, int vdim, int ranges, float eps,
                                  SP_SEQ_PARAMS, int dtype, void* stream) {
  SP_CHECK_ARG(batch_size >= 0 && num_tokens >= 0 && heads > 0 && kv_heads > 0 && heads % kv_heads == 0 && dim > 0 && vdim > 0);
  if (batch_size == 0 || num_tokens == 0) return SP_OK;
  SP_CHECK_ARG(out && q && k && v && gate && pre && dt_bias && A_log && norm_w && state && req_pool_indices && seq_lens);
  SP_CHECK_ARG(!extend_seq_lens || (extend_prefix_lens && extend_start_loc));
  SP_CHECK_ARG(extend_seq_lens || num_tokens == batch_size);
  SP_CHECK_ARG(state_stride >= (int64_t)heads * dim * vdim && pre_stride >= 2 * (int64_t)heads);
  SP_CHECK_ARG(q_stride >= (int64_t)kv_heads * dim && k_stride >= (int64_t)kv_heads * dim);
  SP_CHECK_ARG(v_stride >= (int64_t)heads * vdim && out_stride >= (int64_t)heads * vdim && gate_stride >= (int64_t)heads * vdim);
  SP_CHECK_ARG(ranges >= 1 && (ranges == 1 || workspace));
  if (vdim > kHdMaxV || dim > 256 || heads > 65535) return SP_ERR_UNSUPPORTED;
  SEQ_BATCH(s);
  int cols = (vdim + ranges - 1) / ranges;
  cols = (cols + 7) / 8 * 8;                       // whole 16-byte pieces of a row per workgroup
  ranges = (vdim + cols - 1) / cols;
  const int V = dtype == SP_F32 ? 4 : 8;
  const bool vec = dim % V == 0 && vdim % V == 0 && q_stride % V == 0 && k_stride % V == 0 && v_stride % V == 0 &&
                   (((uintptr_t)q | (uintptr_t)k | (uintptr_t)v) & 15) == 0;
  const HeadDelta a{out, ranges > 1 ? workspace : nullptr, q, k, v, gate, pre, dt_bias, A_log, norm_w, state, out_stride, q_stride,
                    k_stride, v_stride, gate_stride, pre_stride, state_stride, heads, kv_heads, dim, vdim, cols, eps};
  hipStream_t st = (hipStream_t)stream;
  if (dim <= 16) SP_DISPATCH_DTYPE(dtype, return (launch_hd<Tag, 16>(a, s, ranges, vec, num_tokens, st)));
  if (dim <= 32) SP_DISPATCH_DTYPE(dtype, return (launch_hd<Tag, 32>(a, s, ranges, vec, num_tokens, st)));
  if (dim <= 64) SP_DISPATCH_DTYPE(dtype, return (launch_hd<Tag, 64>(a, s, ranges, vec, num_tokens, st)));
  if (dim <= 128) SP_DISPATCH_DTYPE(dtype, return (launch_hd<Tag, 128>(a, s, ranges, vec, num_tokens, st)));
  SP_DISPATCH_DTYPE(dtype, return (launch_hd<Tag, 256>(a, s, ranges, vec, num_tokens, st)));
}
