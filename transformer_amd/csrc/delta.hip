// The gated delta rule: per head a matrix state S [dk][dv] that forgets per key channel and is
// corrected, not just added to, by every token:
//
//     S <- diag(g_t) S,   u_t = beta_t (v_t - S^T k_t),   S <- S + k_t u_t^T,   o_t = S^T q_t
//     g_t = exp(-exp(A_h) softplus(z_t + dt_bias)) per key channel, or one for the whole head,
//     beta_t = sigmoid(b_t),
//     q_t, k_t of unit length (q_t times a constant besides); the heads of a group share q and k
//
//   delta_prepare   : unit q and k, their product k.q, decays and step sizes of all tokens at once
//   delta_recurrent : walks a sequence's tokens in order with S in registers (prompts)
//   delta_step      : a step of single tokens in one kernel: decay and gate (low-rank products, or
//                     projections of their own), unit vectors, the state's update, the readout's norm and gate
//
// The readout needs the updated state, but S_new^T q = (g S)^T q + u (k.q): both sums over key
// channels are taken of the decayed state side by side, and the update is no part of the chain
// that the readout waits for.
//
// State, decays, step sizes, unit vectors and sums are float32; tokens are walked in the same order
// however a sequence was cut into steps.
#include "common.h"

__device__ __forceinline__ float dr_sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float dr_softplus(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }

#define DR_UNIT_EPS 1e-6f       // under the root of a vector's length

// ------------------------------------------------------------------ what does not depend on the state
// One workgroup per token; a wave takes units in turn: the G pairs (q, k), then the H decays (HEAD: z
// holds one number per head, in the engine's type, and all heads' decays are one unit).
template <typename T, typename TZ, bool HEAD>
__global__ __launch_bounds__(256) void delta_prepare_kernel(
    const T* __restrict__ qkv, int stride, const TZ* __restrict__ z, int zstride, const float* __restrict__ dt_bias,
    const float* __restrict__ a_log, const T* __restrict__ braw, int bstride, int G, int H, int dk, float qscale,
    float* __restrict__ qn, float* __restrict__ kn, float* __restrict__ decay, float* __restrict__ beta,
    float* __restrict__ kq) {
  const size_t t = blockIdx.x;
  const int wave = threadIdx.x / TA_WAVE, lane = threadIdx.x % TA_WAVE;
  for (int u = wave; u < G + (HEAD ? 1 : H); u += 4) {
    if (u < G) {
      const T* q = qkv + t * stride + u * dk;
      const T* k = q + G * dk;
      float sq = 0.f, sk = 0.f, sx = 0.f;
      for (int c = lane; c < dk; c += TA_WAVE) {
        const float a = to_f32(q[c]), b = to_f32(k[c]);
        sq = fmaf(a, a, sq);
        sk = fmaf(b, b, sk);
        sx = fmaf(a, b, sx);
      }
      sq = wave_sum(sq);
      sk = wave_sum(sk);
      sx = wave_sum(sx);
      const float fq = qscale * rsqrtf(sq + DR_UNIT_EPS), fk = rsqrtf(sk + DR_UNIT_EPS);
      for (int c = lane; c < dk; c += TA_WAVE) {
        qn[(t * G + u) * dk + c] = to_f32(q[c]) * fq;
        kn[(t * G + u) * dk + c] = to_f32(k[c]) * fk;
      }
      if (lane == 0) kq[t * G + u] = sx * fq * fk;
    } else if (HEAD) {
      for (int h = lane; h < H; h += TA_WAVE) {
        decay[t * H + h] = expf(-expf(a_log[h]) * dr_softplus(to_f32(z[t * zstride + h]) + dt_bias[h]));
        beta[t * H + h] = dr_sigmoid(to_f32(braw[t * bstride + h]));
      }
    } else {
      const int h = u - G;
      const float rate = expf(a_log[h]);
      for (int c = lane; c < dk; c += TA_WAVE) {
        const size_t at = (t * H + h) * dk + c;
        decay[at] = expf(-rate * dr_softplus(to_f32(z[t * zstride + h * dk + c]) + dt_bias[h * dk + c]));
      }
      if (lane == 0) beta[t * H + h] = dr_sigmoid(to_f32(braw[t * bstride + h]));
    }
  }
}

// qkv: [nt, stride] rows of [q: G*dk | k: G*dk | ...] behind convolution and activation; z: decay inputs
// without their bias, [nt, H*dk] float32, or with per_head rows, zstride apart, of H numbers in the engine's
// type (dt_bias then holds H, decay is [nt, H]); braw: [nt] rows, bstride apart, of H step-size inputs.
// qn, kn [nt, G, dk], decay [nt, H, dk], beta [nt, H], kq [nt, G]: float32.
extern "C" int ta_delta_prepare(hipStream_t stream, int dtype, const void* qkv, int stride, const void* z,
                                int zstride, int per_head, const float* dt_bias, const float* a_log, const void* braw, int bstride, int nt,
                                int G, int H, int dk, float qscale, float* qn, float* kn, float* decay, float* beta,
                                float* kq) {
  TA_REQUIRE(nt >= 0 && G >= 1 && H >= 1 && H % G == 0 && dk >= 1, "ta_delta_prepare: bad sizes nt=%d heads=%d/%d width %d", nt, H, G, dk);
  TA_REQUIRE(stride >= 2 * G * dk && bstride >= H && zstride >= (per_head ? H : H * dk), "ta_delta_prepare: rows of %d / %d are too short", stride, bstride);
  if (nt == 0) return 0;
#define DP_RUN(T, TZ, HD)                                                                                           \
  delta_prepare_kernel<T, TZ, HD><<<nt, 256, 0, stream>>>((const T*)qkv, stride, (const TZ*)z, zstride, dt_bias, a_log, \
                                                          (const T*)braw, bstride, G, H, dk, qscale, qn, kn, decay,    \
                                                          beta, kq)
  if (dtype == TA_F32) {
    if (per_head) DP_RUN(float, float, true); else DP_RUN(float, float, false);
  } else if (dtype == TA_BF16) {
    if (per_head) DP_RUN(bf16_t, bf16_t, true); else DP_RUN(bf16_t, float, false);
  } else return ta_fail("ta_delta_prepare: unknown dtype %d", dtype);
#undef DP_RUN
  return ta_check_launch("ta_delta_prepare");
}

// ------------------------------------------------------------------ prompts
// LANES (16 or 32) lanes share a value column, each with R of its key channels (in runs of four: run i of
// lane l holds channels 4 LANES i + 4 l ..+3, so that a wave's operand reads from LDS meet every bank once);
// a wave owns 64 / LANES columns. A token costs a wave some 5 R + 20 vector instructions, and a wave alone on
// its SIMD issues one every five cycles or so: with few heads and sequences 32 lanes share a column, which
// shortens the walk; with many, 16 lanes waste less on the exchange. Operands of the next chunk of tokens
// are on their way to registers while this chunk is worked on out of one of two LDS buffers, and the next
// token's leave LDS a token ahead.
#define DR_FEW_COLUMNS 3072

// HEAD: one decay per token and head, [nt, H]; it travels with the step size.
template <typename T, int LANES, int R, bool VEC, bool HEAD>
__global__ __launch_bounds__(256) void delta_recurrent_kernel(
    const float* __restrict__ qn, const float* __restrict__ kn, const float* __restrict__ decay,
    const T* __restrict__ v, int v_stride, const float* __restrict__ beta, const float* __restrict__ kq,
    float* __restrict__ state, const int* __restrict__ cu_q, const int* __restrict__ slots, int H, int G, int dk,
    int dv, float* __restrict__ o_out) {
  constexpr int DKP = LANES * R, NT = 256, COLS = NT / LANES;
  constexpr int TC = DKP <= 128 ? 16 : 8;          // tokens of a chunk (at most LANES: see `kept`)
  constexpr int NF = (TC * DKP / 4 + NT - 1) / NT; // runs of four that a thread brings in of each operand
  __shared__ __attribute__((aligned(16))) float sq[2][TC][DKP], sk[2][TC][DKP], sg[2][HEAD ? 1 : TC][DKP];
  __shared__ float sv[2][NT / COLS][COLS];         // TC rows are used
  __shared__ float2 sbx[2][TC];                    // step size, k . q
  __shared__ float sgh[2][TC];                     // the head's decay (HEAD)
  const int h = blockIdx.x, col0 = blockIdx.y * COLS, b = blockIdx.z;
  const int start = cu_q[b], end = cu_q[b + 1];
  if (start >= end) return;
  const int g = h / (H / G);
  const int tid = threadIdx.x, lane = tid % LANES, cl = tid / LANES;
  const int col = col0 + cl;
  float* st = state + ((size_t)slots[b] * H + h) * dk * (size_t)dv;
  float S[R];
#pragma unroll
  for (int i = 0; i < R; ++i) {
    const int row = 4 * LANES * (i / 4) + 4 * lane + i % 4;
    S[i] = (row < dk && col < dv) ? st[(size_t)row * dv + col] : 0.f;
  }
  struct Chunk {
    float4 q[NF], k[NF], g[HEAD ? 1 : NF];
    T v;
    float b, x, gh;
  };
  // Every load is issued without a condition (a channel past dk, a column past dv, a token past the
  // sequence's end read what is there and are replaced or not used), so that none is waited for before
  // its chunk goes to LDS. Offsets fit 32 bits (checked on the host).
  auto run4 = [&](const float* p, uint32_t at, int c) {
    if (VEC) return *reinterpret_cast<const float4*>(p + at + (c < dk ? c : 0));
    return float4{p[at + (c < dk ? c : 0)], p[at + (c + 1 < dk ? c + 1 : 0)], p[at + (c + 2 < dk ? c + 2 : 0)],
                  p[at + (c + 3 < dk ? c + 3 : 0)]};
  };
  const uint32_t qstep = (uint32_t)(G * dk), gstep = (uint32_t)(H * dk);
  auto fetch = [&](Chunk& f, int t0) {
#pragma unroll
    for (int e = 0; e < NF; ++e) {
      const int idx = tid + NT * e;
      const int tt = idx / (DKP / 4), c = (idx % (DKP / 4)) * 4;
      const uint32_t t = t0 + tt < end ? t0 + tt : end - 1;
      f.q[e] = run4(qn, t * qstep + g * dk, c);
      f.k[e] = run4(kn, t * qstep + g * dk, c);
      if (!HEAD) f.g[e] = run4(decay, t * gstep + h * dk, c);
    }
    {
      const int c = col0 + tid % COLS;
      const uint32_t t = t0 + tid / COLS < end ? t0 + tid / COLS : end - 1;
      f.v = v[t * (size_t)v_stride + h * dv + (c < dv ? c : 0)];
    }
    const uint32_t t = t0 + tid % TC < end ? t0 + tid % TC : end - 1;
    f.b = beta[t * (uint32_t)H + h];
    f.x = kq[t * (uint32_t)G + g];
    f.gh = HEAD ? decay[t * (uint32_t)H + h] : 1.f;
  };
  auto stash = [&](const Chunk& f, int buf) {
#pragma unroll
    for (int e = 0; e < NF; ++e) {
      const int idx = tid + NT * e, c = (idx % (DKP / 4)) * 4;
      if (TC * DKP / 4 % NT == 0 || idx < TC * DKP / 4) {
        float4 q = f.q[e], k = f.k[e], w = f.g[HEAD ? 0 : e];
        if (c + 4 > dk) {                                     // channels past dk: nothing to read or write, no decay
          if (c + 0 >= dk) { q.x = k.x = 0.f; w.x = 1.f; }
          if (c + 1 >= dk) { q.y = k.y = 0.f; w.y = 1.f; }
          if (c + 2 >= dk) { q.z = k.z = 0.f; w.z = 1.f; }
          q.w = k.w = 0.f;
          w.w = 1.f;
        }
        reinterpret_cast<float4*>(&sq[buf][0][0])[idx] = q;
        reinterpret_cast<float4*>(&sk[buf][0][0])[idx] = k;
        if (!HEAD) reinterpret_cast<float4*>(&sg[buf][0][0])[idx] = w;
      }
    }
    (&sv[buf][0][0])[tid] = to_f32(f.v);
    sbx[buf][tid % TC] = float2{f.b, f.x};                    // (several threads write the same)
    if (HEAD) sgh[buf][tid % TC] = f.gh;
  };
  struct Token {
    float4 q[R / 4], k[R / 4], g[HEAD ? 1 : R / 4];
    float v, gh;
    float2 bx;
  };
  auto take = [&](Token& o, int buf, int tt) {
    if (tt > TC - 1) tt = TC - 1;                           // past the chunk: not used
#pragma unroll
    for (int i = 0; i < R / 4; ++i) {
      if (!HEAD) o.g[i] = *reinterpret_cast<const float4*>(&sg[buf][tt][4 * LANES * i + 4 * lane]);
      o.k[i] = *reinterpret_cast<const float4*>(&sk[buf][tt][4 * LANES * i + 4 * lane]);
      o.q[i] = *reinterpret_cast<const float4*>(&sq[buf][tt][4 * LANES * i + 4 * lane]);
    }
    o.v = sv[buf][tt][cl];
    o.bx = sbx[buf][tt];
    o.gh = HEAD ? sgh[buf][tt] : 1.f;
  };
  float kept = 0.f;                     // lane l keeps the readout of the chunk's token l
  auto token = [&](const Token& o, int tt) {
    float w[4] = {0.f, 0.f, 0.f, 0.f}, r[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < R / 4; ++i) {
      const float4 g4 = o.g[HEAD ? 0 : i];
      const float gs[4] = {g4.x, g4.y, g4.z, g4.w};
      const float ks[4] = {o.k[i].x, o.k[i].y, o.k[i].z, o.k[i].w};
      const float qs[4] = {o.q[i].x, o.q[i].y, o.q[i].z, o.q[i].w};
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        S[4 * i + e] *= HEAD ? o.gh : gs[e];
        w[e] = fmaf(S[4 * i + e], ks[e], w[e]);
        r[e] = fmaf(S[4 * i + e], qs[e], r[e]);
      }
    }
    float ws = (w[0] + w[1]) + (w[2] + w[3]), rs = (r[0] + r[1]) + (r[2] + r[3]);
    ta_sums2<LANES>(ws, rs);
    const float u = o.bx.x * (o.v - ws);
#pragma unroll
    for (int i = 0; i < R / 4; ++i) {
      S[4 * i + 0] = fmaf(o.k[i].x, u, S[4 * i + 0]);
      S[4 * i + 1] = fmaf(o.k[i].y, u, S[4 * i + 1]);
      S[4 * i + 2] = fmaf(o.k[i].z, u, S[4 * i + 2]);
      S[4 * i + 3] = fmaf(o.k[i].w, u, S[4 * i + 3]);
    }
    const float out = fmaf(u, o.bx.y, rs);
    kept = lane == tt ? out : kept;
  };
  {
    Chunk f{};
    fetch(f, start);
    stash(f, 0);
  }
  __syncthreads();
  int buf = 0;
  for (int t0 = start; t0 < end; t0 += TC, buf ^= 1) {
    const int n = end - t0 < TC ? end - t0 : TC;
    Chunk f{};
    fetch(f, t0 + TC);                  // behind the last chunk: its last token again, for nothing
    Token a{}, c{};
    // the next token's operands are asked for in front of this token's arithmetic, and stay there
    __builtin_amdgcn_sched_barrier(0);
    take(a, buf, 0);
    if (n == TC) {
#pragma unroll
      for (int tt = 0; tt < TC; tt += 2) {
        take(c, buf, tt + 1);
        __builtin_amdgcn_sched_barrier(0);
        token(a, tt);
        __builtin_amdgcn_sched_barrier(0);
        if (tt + 2 < TC) take(a, buf, tt + 2);
        __builtin_amdgcn_sched_barrier(0);
        token(c, tt + 1);
        __builtin_amdgcn_sched_barrier(0);
      }
    } else {
      for (int tt = 0; tt < n; ++tt) {
        token(a, tt);
        take(a, buf, tt + 1);
      }
    }
    if (lane < n && col < dv) o_out[((size_t)(t0 + lane) * H + h) * dv + col] = kept;
    // the other buffer's readers are behind the barrier at the end of the turn before
    stash(f, buf ^ 1);
    __syncthreads();
  }
#pragma unroll
  for (int i = 0; i < R; ++i) {
    const int row = 4 * LANES * (i / 4) + 4 * lane + i % 4;
    if (row < dk && col < dv) st[(size_t)row * dv + col] = S[i];
  }
}

// qn, kn, decay, beta, kq: what ta_delta_prepare left. v: [nt] rows, v_stride apart, of H*dv values in
// the engine's type. state [slots, H, dk, dv] float32; o_out [nt, H, dv] float32. lanes that share a value
// column (16 or 32; 0: chosen by the number of heads and sequences). per_head: decay is [nt, H].
extern "C" int ta_delta_recurrent(hipStream_t stream, int dtype, const float* qn, const float* kn, const float* decay,
                                  const void* v, int v_stride, const float* beta, const float* kq, float* state,
                                  const int* cu_q, const int* slots, int batch, int nt, int H, int G, int dk, int dv,
                                  int lanes, int per_head, float* o_out) {
  TA_REQUIRE(batch > 0 && batch <= 65535 && nt >= batch, "ta_delta_recurrent: bad batch %d / tokens %d", batch, nt);
  TA_REQUIRE(G >= 1 && H >= 1 && H % G == 0 && dk >= 1 && dk <= 256 && dv >= 1 && v_stride >= H * dv,
             "ta_delta_recurrent: %d heads in %d groups of %d / %d", H, G, dk, dv);
  TA_REQUIRE(lanes == 0 || lanes == 16 || lanes == 32, "ta_delta_recurrent: %d lanes", lanes);
  TA_REQUIRE((long long)nt * H * dk < (1ll << 31), "ta_delta_recurrent: %d tokens of %d heads of %d in one step", nt, H, dk);
  TA_REQUIRE(dtype == TA_F32 || dtype == TA_BF16, "ta_delta_recurrent: unknown dtype %d", dtype);
  // 32 lanes a column while that leaves a SIMD no more than about two waves
  if (lanes == 0) lanes = (long long)batch * H * dv > DR_FEW_COLUMNS ? 16 : 32;
  if (dk <= 64) lanes = 16;
  const int cols = 256 / lanes;
  TA_REQUIRE((dv + cols - 1) / cols <= 65535, "ta_delta_recurrent: values of %d", dv);
  dim3 g(H, (dv + cols - 1) / cols, batch);
  const bool vec = dk % 4 == 0 && (((uintptr_t)qn | (uintptr_t)kn | (per_head ? 0 : (uintptr_t)decay)) & 15) == 0;
#define DR_RUN(T, L, RR, VE, HD)                                                                          \
  delta_recurrent_kernel<T, L, RR, VE, HD><<<g, 256, 0, stream>>>(qn, kn, decay, (const T*)v, v_stride, beta, kq, \
                                                              state, cu_q, slots, H, G, dk, dv, o_out)
#define DR_BY_VEC(T, L, RR) \
  if (per_head) { if (vec) DR_RUN(T, L, RR, true, true); else DR_RUN(T, L, RR, false, true); } \
  else { if (vec) DR_RUN(T, L, RR, true, false); else DR_RUN(T, L, RR, false, false); }
#define DR_BY_WIDTH(T)                                                  \
  if (dk <= 64) { DR_BY_VEC(T, 16, 4); }                                \
  else if (dk <= 128) {                                                 \
    if (lanes == 32) { DR_BY_VEC(T, 32, 4); } else { DR_BY_VEC(T, 16, 8); } \
  } else {                                                              \
    if (lanes == 32) { DR_BY_VEC(T, 32, 8); } else { DR_BY_VEC(T, 16, 16); } \
  }
  if (dtype == TA_F32) { DR_BY_WIDTH(float) } else { DR_BY_WIDTH(bf16_t) }
#undef DR_BY_WIDTH
#undef DR_BY_VEC
#undef DR_RUN
  return ta_check_launch("ta_delta_recurrent");
}

// ------------------------------------------------------------------ steps of single tokens
// One workgroup of DS_NT threads per (head, sequence). A thread keeps VW neighbouring value columns of
// every RG-th key channel in registers; the state is asked for first, and everything else (unit vectors,
// low-rank products) is formed while it is on its way.
#define DS_NT 512

template <typename T>
__device__ __forceinline__ void ds_load8(const T* p, float* o);
template <>
__device__ __forceinline__ void ds_load8<float>(const float* p, float* o) {
  const float4 a = *reinterpret_cast<const float4*>(p), b = *reinterpret_cast<const float4*>(p + 4);
  o[0] = a.x; o[1] = a.y; o[2] = a.z; o[3] = a.w; o[4] = b.x; o[5] = b.y; o[6] = b.z; o[7] = b.w;
}
template <>
__device__ __forceinline__ void ds_load8<bf16_t>(const bf16_t* p, float* o) {
  const uint4 r = *reinterpret_cast<const uint4*>(p);
  const uint32_t w[4] = {r.x, r.y, r.z, r.w};
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    o[2 * i] = __uint_as_float(w[i] << 16);
    o[2 * i + 1] = __uint_as_float(w[i] & 0xffff0000u);
  }
}

// The product of a weight row with a low-rank input in LDS, four lanes a row (all four get the sum).
template <typename TW>
__device__ __forceinline__ float ds_row_dot(const TW* __restrict__ w, const float* low, int rank, int part, bool vec) {
  float s = 0.f;
  if (vec) {
    for (int r = 8 * part; r < rank; r += 32) {
      float a[8];
      ds_load8<TW>(w + r, a);
#pragma unroll
      for (int e = 0; e < 8; ++e) s = fmaf(a[e], low[r + e], s);
    }
  } else {
    for (int r = part; r < rank; r += 4) s = fmaf(to_f32(w[r]), low[r], s);
  }
  s += __shfl_xor(s, 1, TA_WAVE);
  s += __shfl_xor(s, 2, TA_WAVE);
  return s;
}

template <typename T, typename TW, int VW, int ROWS>
__global__ __launch_bounds__(DS_NT) void delta_step_kernel(
    const T* __restrict__ qkv, int stride, const T* __restrict__ proj, int pstride, int aoff, int ra, int goff, int rg,
    int boff, const TW* __restrict__ a2, const TW* __restrict__ g2, const float* __restrict__ dt_bias,
    const float* __restrict__ a_log, float* __restrict__ state, const int* __restrict__ slots, int H, int G, int dk,
    int dv, float qscale, const float* __restrict__ norm_w, float eps, int a_vec, int g_vec, int gate_act,
    T* __restrict__ out) {
  extern __shared__ float lds[];
  const int CV = dv / VW, RG = DS_NT / CV;           // column groups; row groups
  float* qs = lds;                                   // [dk]
  float* ks = qs + dk;                               // [dk]
  float* gs = ks + dk;                               // [dk]
  float* gate = gs + dk;                             // [dv]
  float* us = gate + dv;                             // [dv]
  float* la = us + dv;                               // [ra]
  float* lg = la + ra;                               // [rg]
  float* pw = lg + rg;                               // [RG][dv]
  float* pr = pw + RG * dv;                          // [RG][dv]
  __shared__ float red[DS_NT / TA_WAVE];
  const int h = blockIdx.x, b = blockIdx.y, tid = threadIdx.x;
  const int kvh = h / (H / G);
  float* st = state + ((size_t)slots[b] * H + h) * dk * (size_t)dv;
  const int r0 = tid / CV, c0 = (tid % CV) * VW;
  const bool on = r0 < RG;
  float S[ROWS][VW];
#pragma unroll
  for (int i = 0; i < ROWS; ++i) {
    const int row = r0 + RG * i;
    const bool ok = on && row < dk;
    const float* p = st + (size_t)(ok ? row : 0) * dv + c0;
    if (VW == 4) {
      const float4 a = *reinterpret_cast<const float4*>(p);
      S[i][0] = ok ? a.x : 0.f;
      S[i][VW > 1 ? 1 : 0] = VW > 1 ? (ok ? a.y : 0.f) : S[i][0];
      S[i][VW > 2 ? 2 : 0] = VW > 2 ? (ok ? a.z : 0.f) : S[i][0];
      S[i][VW > 3 ? 3 : 0] = VW > 3 ? (ok ? a.w : 0.f) : S[i][0];
    } else {
      const float a = p[0];
      S[i][0] = ok ? a : 0.f;
    }
  }
  // ---- operands to LDS
  const T* row = qkv + (size_t)b * stride;
  for (int c = tid; c < dk; c += DS_NT) {
    qs[c] = to_f32(row[kvh * dk + c]);
    ks[c] = to_f32(row[(G + kvh) * dk + c]);
  }
  const T* prow = proj + (size_t)b * pstride;
  for (int c = tid; c < ra; c += DS_NT) la[c] = to_f32(prow[aoff + c]);
  for (int c = tid; c < rg; c += DS_NT) lg[c] = to_f32(prow[goff + c]);
  const float beta = dr_sigmoid(to_f32(prow[boff + h]));
  const float rate = expf(a_log[h]);
  __syncthreads();
  // ---- factors of the unit vectors (every wave for itself), decays, output gates
  float sq = 0.f, sk = 0.f, sx = 0.f;
  for (int c = tid % TA_WAVE; c < dk; c += TA_WAVE) {
    const float a = qs[c], k = ks[c];
    sq = fmaf(a, a, sq);
    sk = fmaf(k, k, sk);
    sx = fmaf(a, k, sx);
  }
  sq = wave_sum(sq);
  sk = wave_sum(sk);
  sx = wave_sum(sx);
  const float fq = qscale * rsqrtf(sq + DR_UNIT_EPS), fk = rsqrtf(sk + DR_UNIT_EPS);
  const float kq = sx * fq * fk;
  auto gate_of = [&](float z) { return gate_act == 1 ? dr_sigmoid(z) : z * dr_sigmoid(z); };
  if (ra == 0) {                                     // one decay for the head
    const float g = expf(-rate * dr_softplus(to_f32(prow[aoff + h]) + dt_bias[h]));
    for (int c = tid; c < dk; c += DS_NT) gs[c] = g;
  }
  if (rg == 0)                                       // the gate as projected
    for (int j = tid; j < dv; j += DS_NT) gate[j] = gate_of(to_f32(prow[goff + h * dv + j]));
  // (whole groups of four lanes take a row; the loop's bound is the same for the four)
  for (int i = tid / 4 + (ra == 0 ? dk : 0); i < (rg == 0 ? dk : dk + dv); i += DS_NT / 4) {
    const bool dec = i < dk;
    const int j = dec ? i : i - dk;
    const float s = dec ? ds_row_dot<TW>(a2 + ((size_t)h * dk + j) * ra, la, ra, tid % 4, a_vec)
                        : ds_row_dot<TW>(g2 + ((size_t)h * dv + j) * rg, lg, rg, tid % 4, g_vec);
    if (tid % 4 == 0) {
      if (dec) gs[j] = expf(-rate * dr_softplus(s + dt_bias[h * dk + j]));
      else gate[j] = gate_of(s);
    }
  }
  __syncthreads();
  // ---- the decayed state and its products with k and q
  float w[VW], r[VW];
#pragma unroll
  for (int e = 0; e < VW; ++e) w[e] = r[e] = 0.f;
#pragma unroll
  for (int i = 0; i < ROWS; ++i) {
    const int rw = r0 + RG * i;
    const bool ok = on && rw < dk;
    const float g = gs[ok ? rw : 0], k = ks[ok ? rw : 0] * fk, q = qs[ok ? rw : 0] * fq;
#pragma unroll
    for (int e = 0; e < VW; ++e) {
      S[i][e] *= g;
      w[e] = fmaf(S[i][e], k, w[e]);
      r[e] = fmaf(S[i][e], q, r[e]);
    }
  }
  if (on) {
#pragma unroll
    for (int e = 0; e < VW; ++e) {
      pw[r0 * dv + c0 + e] = w[e];
      pr[r0 * dv + c0 + e] = r[e];
    }
  }
  __syncthreads();
  float ss = 0.f;
  const T* vrow = row + 2 * G * dk + (size_t)h * dv;
  for (int j = tid; j < dv; j += DS_NT) {            // row groups in order
    float ws = 0.f, rs = 0.f;
    for (int i = 0; i < RG; ++i) {
      ws += pw[i * dv + j];
      rs += pr[i * dv + j];
    }
    const float u = beta * (to_f32(vrow[j]) - ws);
    const float o = fmaf(u, kq, rs);
    us[j] = u;
    pr[j] = o;                                       // column j of row group 0 is this thread's alone now
    ss = fmaf(o, o, ss);
  }
  ss = wave_sum(ss);
  if (tid % TA_WAVE == 0) red[tid / TA_WAVE] = ss;
  __syncthreads();
  // ---- the update
#pragma unroll
  for (int i = 0; i < ROWS; ++i) {
    const int rw = r0 + RG * i;
    if (on && rw < dk) {
      const float k = ks[rw] * fk;
      float n[VW];
#pragma unroll
      for (int e = 0; e < VW; ++e) n[e] = fmaf(k, us[c0 + e], S[i][e]);
      float* p = st + (size_t)rw * dv + c0;
      if (VW == 4) *reinterpret_cast<float4*>(p) = float4{n[0], n[VW > 1 ? 1 : 0], n[VW > 2 ? 2 : 0], n[VW > 3 ? 3 : 0]};
      else p[0] = n[0];
    }
  }
  // ---- the readout's norm and gate
  float tot = 0.f;
#pragma unroll
  for (int i = 0; i < DS_NT / TA_WAVE; ++i) tot += red[i];
  const float f = rsqrtf(tot / (float)dv + eps);
  for (int j = tid; j < dv; j += DS_NT)
    out[(size_t)b * H * dv + (size_t)h * dv + j] = from_f32<T>(pr[j] * f * norm_w[j] * gate[j]);
}

static int delta_step_rows(int dk, int dv) {          // key channels a thread keeps; 0: not taken
  const int cv = dv % 4 == 0 ? dv / 4 : dv;
  if (cv < 1 || cv > DS_NT) return 0;
  const int rg = DS_NT / cv;
  const int rows = (dk + rg - 1) / rg;
  return rows <= 4 ? 4 : rows <= 8 ? 8 : rows <= 16 ? 16 : rows <= 32 ? 32 : 0;
}
static size_t delta_step_lds(int dk, int dv, int ra, int rg) {
  const int cv = dv % 4 == 0 ? dv / 4 : dv;
  return ((size_t)3 * dk + 2 * dv + ra + rg + (size_t)2 * (DS_NT / cv) * dv) * sizeof(float);
}

// Whether ta_delta_step takes heads of dk x dv with low-rank inputs of ra and rg (0: none).
extern "C" int ta_delta_step_fits(int dk, int dv, int ra, int rg) {
  return dk >= 1 && ra >= 0 && rg >= 0 && delta_step_rows(dk, dv) > 0 && delta_step_lds(dk, dv, ra, rg) <= 60000;
}

// qkv: [batch] rows, stride apart, of [q: G*dk | k: G*dk | v: H*dv] behind convolution and activation;
// proj: [batch] rows, pstride apart, holding the decay's low-rank input (ra) at aoff, the gate's (rg) at
// goff and the step sizes' (H) at boff; a2 [H*dk, ra], g2 [H*dv, rg]; state [slots, H, dk, dv] float32;
// norm_w [dv]; out [batch, H*dv] = the readout over its root mean square per head, times norm_w, gated
// (gate_act 0: silu, 1: sigmoid). ra 0: the rows hold H decay inputs at aoff, one per head, and dt_bias H
// numbers; rg 0: they hold the gates (H*dv) at goff.
extern "C" int ta_delta_step(hipStream_t stream, int dtype, int wdtype, const void* qkv, int stride, const void* proj,
                             int pstride, int aoff, int ra, int goff, int rg, int boff, const void* a2, const void* g2,
                             const float* dt_bias, const float* a_log, float* state, const int* slots, int batch, int H,
                             int G, int dk, int dv, float qscale, const float* norm_w, float eps, int gate_act,
                             void* out) {
  TA_REQUIRE(batch > 0 && batch <= 65535 && G >= 1 && H >= 1 && H % G == 0, "ta_delta_step: batch %d, %d heads in %d groups", batch, H, G);
  TA_REQUIRE(ta_delta_step_fits(dk, dv, ra, rg), "ta_delta_step: heads of %d x %d, ranks %d / %d", dk, dv, ra, rg);
  TA_REQUIRE(stride >= 2 * G * dk + H * dv && aoff >= 0 && goff >= 0 && boff >= 0 &&
             pstride >= aoff + (ra ? ra : H) && pstride >= goff + (rg ? rg : H * dv) && pstride >= boff + H, "ta_delta_step: rows of %d / %d are too short", stride, pstride);
  TA_REQUIRE(gate_act == 0 || gate_act == 1, "ta_delta_step: unknown gate activation %d", gate_act);
  const int rows = delta_step_rows(dk, dv);
  const size_t lds = delta_step_lds(dk, dv, ra, rg);
  const int a_vec = ra % 8 == 0 && (uintptr_t)a2 % 16 == 0, g_vec = rg % 8 == 0 && (uintptr_t)g2 % 16 == 0;
  const bool wide = dv % 4 == 0 && (uintptr_t)state % 16 == 0;
  TA_REQUIRE(wide || dv % 4 != 0, "ta_delta_step: the state must be 16-byte aligned");
  dim3 g(H, batch);
#define DS_RUN(T, TW, VWV, RW)                                                                                       \
  delta_step_kernel<T, TW, VWV, RW><<<g, DS_NT, lds, stream>>>(                                                      \
      (const T*)qkv, stride, (const T*)proj, pstride, aoff, ra, goff, rg, boff, (const TW*)a2, (const TW*)g2, dt_bias, \
      a_log, state, slots, H, G, dk, dv, qscale, norm_w, eps, a_vec, g_vec, gate_act, (T*)out)
#define DS_BY_ROWS(T, TW, VWV)                 \
  switch (rows) {                              \
    case 4: DS_RUN(T, TW, VWV, 4); break;      \
    case 8: DS_RUN(T, TW, VWV, 8); break;      \
    case 16: DS_RUN(T, TW, VWV, 16); break;    \
    default: DS_RUN(T, TW, VWV, 32); break;    \
  }
#define DS_BY_COLS(T, TW) \
  if (wide) { DS_BY_ROWS(T, TW, 4) } else { DS_BY_ROWS(T, TW, 1) }
  if (dtype == TA_F32 && wdtype == TA_F32) { DS_BY_COLS(float, float) }
  else if (dtype == TA_BF16 && wdtype == TA_BF16) { DS_BY_COLS(bf16_t, bf16_t) }
  else if (dtype == TA_BF16 && wdtype == TA_F32) { DS_BY_COLS(bf16_t, float) }
  else return ta_fail("ta_delta_step: unsupported dtypes %d / %d", dtype, wdtype);
#undef DS_BY_COLS
#undef DS_BY_ROWS
#undef DS_RUN
  return ta_check_launch("ta_delta_step");
}
