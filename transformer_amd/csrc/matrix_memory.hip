// The matrix memory of xLSTM ("mLSTM"): per head a state S [dk][dv], a normaliser n [dk] and a running
// maximum m (0 at a sequence's start), with exponential gates that are kept as logarithms:
//
//     i_t = cap tanh((a_t + bi) / cap),  f_t = log sigmoid(cap tanh((b_t + bf) / cap))
//     m_t = max(f_t + m_(t-1), i_t),  keep_t = exp(f_t + m_(t-1) - m_t),  write_t = exp(i_t - m_t)
//     S_t = keep_t S_(t-1) + write_t k_t v_t^T,  n_t = keep_t n_(t-1) + write_t k_t
//     o_t = S_t^T q_t / (max(|n_t . q_t|, exp(-m_t)) + 1e-6)
//
//   memory_gates : keep, write and exp(-m) of every token and head; the running maximum by a scan over
//                  the waves of a workgroup
//   memory_recurrent : walks a sequence's tokens in order with S in registers; the normaliser is one more value
//                  column whose value is always 1
//   memory_step  : a step of single tokens in one kernel: gates, the state's update, the readout with its
//                  denominator, the head's norm and the output gate; heads too large for one workgroup take
//                  two kernels, the second of which moves normaliser and maximum on and does what needs the whole
//                  readout
//
// keep is formed as exp(f - (m_t - m_(t-1))): where m_t is the rounded f + m_(t-1), the difference of the
// two maxima is exact and keep makes up for that rounding.
#include "common.h"

#define MM_FLOOR_EPS 1e-6f      // beside the denominator

__device__ __forceinline__ float mm_cap(float z, float cap) { return cap * tanhf(z / cap); }
__device__ __forceinline__ float mm_log_sigmoid(float z) { return fminf(z, 0.f) - log1pf(expf(-fabsf(z))); }

// ------------------------------------------------------------------ gates of a step
// One workgroup of WAVES waves per (head, sequence), a token a thread. Elements of the scan are (sum of f, best
// of i_j + f_(j+1) + .. + f_t); two neighbours join to (F1 + F2, max(M1 + F2, M2)), and m_t = max(F + m before
// the turn, M). A wave scans its 64 tokens; the waves' totals are joined in order by every wave for itself.
template <typename T, int WAVES>
__global__ __launch_bounds__(WAVES * TA_WAVE) void memory_gates_kernel(
    const T* __restrict__ proj, int stride, int ioff, int foff, const float* __restrict__ ibias,
    const float* __restrict__ fbias, float cap, float* __restrict__ m_state, const int* __restrict__ cu_q,
    const int* __restrict__ slots, int H, float* __restrict__ keep, float* __restrict__ write, float* __restrict__ floor_) {
  constexpr int NT = WAVES * TA_WAVE;
  __shared__ float2 total[2][WAVES];                // a turn's waves: sum of f, best
  const int h = blockIdx.x, b = blockIdx.y, lane = threadIdx.x % TA_WAVE, wave = threadIdx.x / TA_WAVE;
  const int start = cu_q[b], end = cu_q[b + 1];
  if (start >= end) return;
  float* ms = m_state + (size_t)slots[b] * H + h;
  float m0 = *ms;
  const float bi = ibias[h], bf = fbias[h];
  // the next turn's inputs are on their way while this turn is worked on
  auto at = [&](int t) { return (size_t)(t < end ? t : end - 1) * stride; };
  T ri = proj[at(start + threadIdx.x) + ioff + h], rf = proj[at(start + threadIdx.x) + foff + h];
  int buf = 0;
  for (int t0 = start; t0 < end; t0 += NT, buf ^= 1) {
    const int t = t0 + threadIdx.x;
    const bool on = t < end;
    const float i = on ? mm_cap(to_f32(ri) + bi, cap) : -INFINITY;
    const float f = on ? mm_log_sigmoid(mm_cap(to_f32(rf) + bf, cap)) : 0.f;
    if (t0 + NT < end) {
      ri = proj[at(t + NT) + ioff + h];
      rf = proj[at(t + NT) + foff + h];
    }
    float F = f, M = i;
#pragma unroll
    for (int o = 1; o < TA_WAVE; o <<= 1) {
      const float Fp = __shfl_up(F, o, TA_WAVE), Mp = __shfl_up(M, o, TA_WAVE);
      if (lane >= o) {
        M = fmaxf(Mp + F, M);
        F += Fp;
      }
    }
    float mine = m0;                                // the maximum in front of this wave's tokens
    if (WAVES > 1) {
      if (lane == TA_WAVE - 1) total[buf][wave] = float2{F, M};
      __syncthreads();                              // (a buffer's readers are behind the next turn's barrier)
      float run = m0;
#pragma unroll
      for (int w = 0; w < WAVES; ++w) {
        if (w == wave) mine = run;
        const float2 e = total[buf][w];
        run = fmaxf(e.x + run, e.y);
      }
      m0 = run;
    }
    const float m = fmaxf(F + mine, M);
    const float up = __shfl_up(m, 1, TA_WAVE);
    const float before = lane == 0 ? mine : up;
    if (on) {
      const size_t e = (size_t)t * H + h;
      keep[e] = expf(f - (m - before));
      write[e] = expf(i - m);
      floor_[e] = expf(-m);
    }
    if (WAVES == 1) m0 = __shfl(m, TA_WAVE - 1, TA_WAVE);       // (lanes past the end carry the last token's)
  }
  if (threadIdx.x == 0) *ms = m0;
}

// proj: [nt] rows, stride apart, with the input gates' numbers (H) at column ioff and the forget gates' at
// foff; ibias, fbias [H]; m_state [slots, H] float32, moved on; keep, write, floor_ [nt, H] float32. max_qlen: the
// most tokens a sequence brings (chooses the launch alone).
extern "C" int ta_memory_gates(hipStream_t stream, int dtype, const void* proj, int stride, int ioff, int foff,
                               const float* ibias, const float* fbias, float cap, float* m_state, const int* cu_q,
                               const int* slots, int batch, int nt, int max_qlen, int H, float* keep, float* write, float* floor_) {
  TA_REQUIRE(batch > 0 && batch <= 65535 && nt >= batch && H >= 1, "ta_memory_gates: batch %d, %d tokens, %d heads", batch, nt, H);
  TA_REQUIRE(ioff >= 0 && foff >= 0 && stride >= ioff + H && stride >= foff + H, "ta_memory_gates: rows of %d are too short", stride);
  TA_REQUIRE(cap > 0.f, "ta_memory_gates: the cap must be positive, got %g", (double)cap);
  dim3 g(H, batch);
#define MG_RUN(T, W)                                                                                               \
  memory_gates_kernel<T, W><<<g, W * TA_WAVE, 0, stream>>>((const T*)proj, stride, ioff, foff, ibias, fbias, cap, \
                                                           m_state, cu_q, slots, H, keep, write, floor_)
#define MG_BY_LEN(T) \
  if (max_qlen <= TA_WAVE) MG_RUN(T, 1); else if (max_qlen <= 4 * TA_WAVE) MG_RUN(T, 4); else MG_RUN(T, 16)
  if (dtype == TA_F32) { MG_BY_LEN(float); }
  else if (dtype == TA_BF16) { MG_BY_LEN(bf16_t); }
  else return ta_fail("ta_memory_gates: unknown dtype %d", dtype);
#undef MG_BY_LEN
#undef MG_RUN
  return ta_check_launch("ta_memory_gates");
}

// ------------------------------------------------------------------ prompts
// LANES (16, 32 or 64) lanes share a value column, each with R of its key channels (in runs of four: run i of lane
// l holds channels 4 LANES i + 4 l ..+3, so that a wave's operand reads from LDS meet every bank once); a wave owns
// 64 / LANES columns. Operands of the next chunk of tokens are on their way to registers while this chunk is worked
// on out of one of two LDS buffers; keys wait in LDS already times their write weight, and the next token's
// operands leave LDS a token ahead. Two tokens' readouts are summed over the lanes together, outside the chain of
// updates.
template <typename T, int LANES, int R, bool VEC>
__global__ __launch_bounds__(256) void memory_recurrent_kernel(
    const T* __restrict__ proj, int stride, int qoff, int koff, int voff, float qscale, const float* __restrict__ keep,
    const float* __restrict__ write, float* __restrict__ state, float* __restrict__ n_state,
    const int* __restrict__ cu_q, const int* __restrict__ slots, int H, int dk, int dv, float* __restrict__ o_out,
    float* __restrict__ den_out) {
  constexpr int DKP = LANES * R, NT = 256, COLS = NT / LANES;
  constexpr int TC = DKP <= 128 ? 16 : 2048 / DKP;   // tokens of a chunk (even, at most LANES: see `kept`)
  constexpr int NF = (TC * DKP / 4 + NT - 1) / NT;   // runs of four that a thread brings in of each operand
  __shared__ __attribute__((aligned(16))) float sq[2][TC][DKP], sk[2][TC][DKP];
  __shared__ float sv[2][TC][COLS];                  // (TC * COLS is at most NT)
  __shared__ float sg[2][TC];
  const int h = blockIdx.x, col0 = blockIdx.y * COLS, b = blockIdx.z;
  const int start = cu_q[b], end = cu_q[b + 1];
  if (start >= end) return;
  const int tid = threadIdx.x, lane = tid % LANES, cl = tid / LANES;
  const int col = col0 + cl;                         // dv: the normaliser
  const size_t head = (size_t)slots[b] * H + h;
  float* st = col < dv ? state + head * dk * (size_t)dv + col : n_state + head * dk;
  const size_t sstep = col < dv ? dv : 1;
  const bool mine = col <= dv;
  float S[R];
#pragma unroll
  for (int i = 0; i < R; ++i) {
    const int row = 4 * LANES * (i / 4) + 4 * lane + i % 4;
    S[i] = (mine && row < dk) ? st[row * sstep] : 0.f;
  }
  struct alignas(4 * sizeof(T)) Run { T x[4]; };
  struct Chunk {
    Run q[NF], k[NF];
    float w[NF], g;
    T v;
  };
  // every load is issued without a condition (a channel past dk, a column past dv, a token past the sequence's
  // end read what is there and are replaced), so that none is waited for before its chunk goes to LDS
  auto run4 = [&](const T* p, int c) {
    if (VEC) return *reinterpret_cast<const Run*>(p + (c < dk ? c : 0));
    Run r;
#pragma unroll
    for (int e = 0; e < 4; ++e) r.x[e] = p[c + e < dk ? c + e : 0];
    return r;
  };
  auto fetch = [&](Chunk& f, int t0) {
#pragma unroll
    for (int e = 0; e < NF; ++e) {
      const int idx = tid + NT * e, tt = idx / (DKP / 4), c = (idx % (DKP / 4)) * 4;
      const size_t t = t0 + tt < end ? t0 + tt : end - 1;
      const T* row = proj + t * stride + h * dk;
      f.q[e] = run4(row + qoff, c);
      f.k[e] = run4(row + koff, c);
      f.w[e] = write[t * H + h];
    }
    {
      const int tt = tid / COLS, c = col0 + tid % COLS;
      const size_t t = t0 + tt < end ? t0 + tt : end - 1;
      f.v = proj[t * stride + voff + h * dv + (c < dv ? c : 0)];
    }
    const size_t t = t0 + tid % TC < end ? t0 + tid % TC : end - 1;
    f.g = keep[t * H + h];
  };
  auto stash = [&](const Chunk& f, int t0, int buf) {
#pragma unroll
    for (int e = 0; e < NF; ++e) {
      const int idx = tid + NT * e, tt = idx / (DKP / 4), c = (idx % (DKP / 4)) * 4;
      if (TC * DKP / 4 % NT == 0 || idx < TC * DKP / 4) {
        const float w = t0 + tt < end ? f.w[e] : 0.f;         // a token past the end writes nothing
        float q[4], k[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          const bool ok = c + j < dk;
          q[j] = ok ? to_f32(f.q[e].x[j]) * qscale : 0.f;
          k[j] = ok ? to_f32(f.k[e].x[j]) * w : 0.f;
        }
        reinterpret_cast<float4*>(&sq[buf][0][0])[idx] = float4{q[0], q[1], q[2], q[3]};
        reinterpret_cast<float4*>(&sk[buf][0][0])[idx] = float4{k[0], k[1], k[2], k[3]};
      }
    }
    if (TC * COLS == NT || tid < TC * COLS) (&sv[buf][0][0])[tid] = col0 + tid % COLS == dv ? 1.f : to_f32(f.v);
    if (tid < TC) sg[buf][tid] = t0 + tid < end ? f.g : 1.f;
  };
  struct Token {
    float4 q[R / 4], k[R / 4];
    float v, g;
  };
  auto take = [&](Token& o, int buf, int tt) {
    if (tt > TC - 1) tt = TC - 1;                             // past the chunk: not used
#pragma unroll
    for (int i = 0; i < R / 4; ++i) {
      o.k[i] = *reinterpret_cast<const float4*>(&sk[buf][tt][4 * LANES * i + 4 * lane]);
      o.q[i] = *reinterpret_cast<const float4*>(&sq[buf][tt][4 * LANES * i + 4 * lane]);
    }
    o.v = sv[buf][tt][cl];
    o.g = sg[buf][tt];
  };
  auto token = [&](const Token& o) {
    float r[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < R / 4; ++i) {
      const float ks[4] = {o.k[i].x, o.k[i].y, o.k[i].z, o.k[i].w};
      const float qs[4] = {o.q[i].x, o.q[i].y, o.q[i].z, o.q[i].w};
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        S[4 * i + e] = fmaf(o.g, S[4 * i + e], ks[e] * o.v);
        r[e] = fmaf(S[4 * i + e], qs[e], r[e]);
      }
    }
    return (r[0] + r[1]) + (r[2] + r[3]);
  };
  float* out = col < dv ? o_out + (size_t)h * dv + col : den_out + h;
  const size_t ostep = col < dv ? (size_t)H * dv : (size_t)H;
  {
    Chunk f;
    fetch(f, start);
    stash(f, start, 0);
  }
  __syncthreads();
  int buf = 0;
  for (int t0 = start; t0 < end; t0 += TC, buf ^= 1) {
    const int n = end - t0 < TC ? end - t0 : TC;
    Chunk f;
    fetch(f, t0 + TC);                  // behind the last chunk: its last token again, for nothing
    float kept = 0.f;                   // lane l keeps the readout of the chunk's token l
    Token a, c;
    // the next token's operands are asked for in front of this token's arithmetic, and stay there
    __builtin_amdgcn_sched_barrier(0);
    take(a, buf, 0);
    auto pair = [&](int tt) {
      take(c, buf, tt + 1);
      __builtin_amdgcn_sched_barrier(0);
      float r0 = token(a);
      __builtin_amdgcn_sched_barrier(0);
      take(a, buf, tt + 2);
      __builtin_amdgcn_sched_barrier(0);
      float r1 = token(c);
      ta_sums2<LANES>(r0, r1);
      kept = lane == tt ? r0 : lane == tt + 1 ? r1 : kept;
    };
    if (n == TC) {
#pragma unroll
      for (int tt = 0; tt < TC; tt += 2) pair(tt);
    } else {
      for (int tt = 0; tt < n; tt += 2) pair(tt);             // (an odd end is filled up with a token that writes nothing)
    }
    if (lane < n && mine) out[(size_t)(t0 + lane) * ostep] = kept;
    // the other buffer's readers are behind the barrier at the end of the turn before
    stash(f, t0 + TC, buf ^ 1);
    __syncthreads();
  }
#pragma unroll
  for (int i = 0; i < R; ++i) {
    const int row = 4 * LANES * (i / 4) + 4 * lane + i % 4;
    if (mine && row < dk) st[row * sstep] = S[i];
  }
}

#define MM_FEW_COLUMNS 4096     // columns (sequences x heads x values) up to which 32 lanes share one
#define MM_MAX_KEY_DIM 1024

// proj: [nt] rows, stride apart, with q and k (H*dk each) and v (H*dv) at columns qoff, koff, voff; q is taken times
// qscale. keep, write [nt, H] (ta_memory_gates); state [slots, H, dk, dv], n_state [slots, H, dk] float32, moved on.
// o_out [nt, H, dv] = S_t^T q_t, den_out [nt, H] = n_t . q_t, float32. lanes that share a column (0: chosen by the
// shape; 16 or 32, where the key width leaves the choice).
extern "C" int ta_memory_recurrent(hipStream_t stream, int dtype, const void* proj, int stride, int qoff, int koff,
                                   int voff, float qscale, const float* keep, const float* write, float* state,
                                   float* n_state, const int* cu_q, const int* slots, int batch, int nt, int H, int dk,
                                   int dv, int lanes, float* o_out, float* den_out) {
  TA_REQUIRE(batch > 0 && batch <= 65535 && nt >= batch && H >= 1, "ta_memory_recurrent: batch %d, %d tokens, %d heads", batch, nt, H);
  TA_REQUIRE(dk >= 1 && dk <= MM_MAX_KEY_DIM && dv >= 1, "ta_memory_recurrent: heads of %d x %d", dk, dv);
  TA_REQUIRE(qoff >= 0 && koff >= 0 && voff >= 0 && stride >= qoff + H * dk && stride >= koff + H * dk &&
             stride >= voff + H * dv, "ta_memory_recurrent: rows of %d are too short", stride);
  TA_REQUIRE(lanes == 0 || lanes == 16 || lanes == 32, "ta_memory_recurrent: %d lanes", lanes);
  TA_REQUIRE(dtype == TA_F32 || dtype == TA_BF16, "ta_memory_recurrent: unknown dtype %d", dtype);
  if (lanes == 0) lanes = (long long)batch * H * dv > MM_FEW_COLUMNS ? 16 : 32;
  if (dk <= 64) lanes = 16;
  if (dk > 256) lanes = 32;
  if (dk > 512) lanes = 64;
  const int cols = 256 / lanes, tiles = (dv + 1 + cols - 1) / cols;
  TA_REQUIRE(tiles <= 65535, "ta_memory_recurrent: values of %d", dv);
  dim3 g(H, tiles, batch);
  const int item = dtype == TA_F32 ? 4 : 2;
  const bool vec = dk % 4 == 0 && qoff % 4 == 0 && koff % 4 == 0 && stride % 4 == 0 && (uintptr_t)proj % (4 * item) == 0;
#define MR_RUN(T, L, RR, VE)                                                                                             \
  memory_recurrent_kernel<T, L, RR, VE><<<g, 256, 0, stream>>>((const T*)proj, stride, qoff, koff, voff, qscale, keep,   \
                                                               write, state, n_state, cu_q, slots, H, dk, dv, o_out, den_out)
#define MR_BY_VEC(T, L, RR) \
  if (vec) MR_RUN(T, L, RR, true); else MR_RUN(T, L, RR, false)
#define MR_BY_WIDTH(T)                                                      \
  if (dk <= 64) { MR_BY_VEC(T, 16, 4); }                                    \
  else if (dk <= 128) {                                                     \
    if (lanes == 32) { MR_BY_VEC(T, 32, 4); } else { MR_BY_VEC(T, 16, 8); }   \
  } else if (dk <= 256) {                                                   \
    if (lanes == 32) { MR_BY_VEC(T, 32, 8); } else { MR_BY_VEC(T, 16, 16); }  \
  } else if (dk <= 512) { MR_BY_VEC(T, 32, 16); }                           \
  else { MR_BY_VEC(T, 64, 16); }
  if (dtype == TA_F32) { MR_BY_WIDTH(float) } else { MR_BY_WIDTH(bf16_t) }
#undef MR_BY_WIDTH
#undef MR_BY_VEC
#undef MR_RUN
  return ta_check_launch("ta_memory_recurrent");
}

// ------------------------------------------------------------------ steps of single tokens
// One workgroup of MS_NT threads per (head, sequence). A thread keeps VW neighbouring value columns of every
// RG-th key channel; the whole state is asked for before anything else is done.
// SPLIT: a workgroup owns dvt of the head's columns, leaves their readout in o_out [batch, H, dv] as it is, and
// changes neither n nor m, which the other workgroups of the head read as well.
#define MS_NT 512

struct MemoryGates {
  float keep, write, m;
};
// of one token, from what stood in m_state before it
template <typename T>
__device__ __forceinline__ MemoryGates mm_gates(const T* __restrict__ row, int ioff, int foff, int h,
                                                const float* __restrict__ ibias, const float* __restrict__ fbias,
                                                float cap, float before) {
  const float i = mm_cap(to_f32(row[ioff + h]) + ibias[h], cap);
  const float f = mm_log_sigmoid(mm_cap(to_f32(row[foff + h]) + fbias[h], cap));
  const float m = fmaxf(f + before, i);
  return MemoryGates{expf(f - (m - before)), expf(i - m), m};
}

template <typename T, int VW, int ROWS, bool SPLIT>
__global__ __launch_bounds__(MS_NT) void memory_step_kernel(
    const T* __restrict__ proj, int stride, int qoff, int koff, int voff, int goff, int ioff, int foff,
    const float* __restrict__ ibias, const float* __restrict__ fbias, float cap, float* __restrict__ state,
    float* __restrict__ n_state, float* __restrict__ m_state, const int* __restrict__ slots, int H, int dk, int dv,
    float qscale, const float* __restrict__ norm_w, float eps, T* __restrict__ out, int dvt, float* __restrict__ o_out) {
  extern __shared__ float lds[];
  const int CV = dvt / VW, RG = MS_NT / CV;          // column groups; row groups
  const int cb = SPLIT ? blockIdx.z * dvt : 0;       // this workgroup's first column and their number
  const int dvc = SPLIT && dv - cb < dvt ? dv - cb : dvt;
  float* qs = lds;                                   // [dk]
  float* ks = qs + dk;                               // [dk], times the write weight
  float* pr = ks + dk;                               // [RG][dvt]
  __shared__ float red[MS_NT / TA_WAVE], redn[MS_NT / TA_WAVE];
  const int h = blockIdx.x, b = blockIdx.y, tid = threadIdx.x;
  const size_t slot = (size_t)slots[b];
  float* st = state + (slot * H + h) * dk * (size_t)dv + cb;
  float* ns = n_state + (slot * H + h) * dk;
  const int r0 = tid / CV, c0 = (tid % CV) * VW;
  const bool on = r0 < RG && c0 < dvc;
  float S[ROWS][VW];
#pragma unroll
  for (int i = 0; i < ROWS; ++i) {
    const int row = r0 + RG * i;
    const bool ok = on && row < dk;
    const float* p = st + (size_t)(ok ? row : 0) * dv + (on ? c0 : 0);
    if (VW == 4) {
      const float4 a = *reinterpret_cast<const float4*>(p);
      S[i][0] = a.x;
      S[i][VW > 1 ? 1 : 0] = VW > 1 ? a.y : S[i][0];
      S[i][VW > 2 ? 2 : 0] = VW > 2 ? a.z : S[i][0];
      S[i][VW > 3 ? 3 : 0] = VW > 3 ? a.w : S[i][0];
    } else {
      S[i][0] = p[0];
    }
  }
  const T* row = proj + (size_t)b * stride;
  float v[VW];
#pragma unroll
  for (int e = 0; e < VW; ++e) v[e] = on ? to_f32(row[voff + h * dv + cb + c0 + e]) : 0.f;
  // the gates, by every thread for itself
  const MemoryGates gt = mm_gates(row, ioff, foff, h, ibias, fbias, cap, m_state[slot * H + h]);
  const float keep = gt.keep, write = gt.write, m = gt.m;
  // the normaliser and its product with q
  float dot = 0.f;
  for (int c = tid; c < dk; c += MS_NT) {
    const float q = to_f32(row[qoff + h * dk + c]) * qscale, k = to_f32(row[koff + h * dk + c]) * write;
    qs[c] = q;
    ks[c] = k;
    if (!SPLIT) {
      const float n = fmaf(keep, ns[c], k);
      ns[c] = n;
      dot = fmaf(n, q, dot);
    }
  }
  if (!SPLIT) {
    dot = wave_sum(dot);
    if (tid % TA_WAVE == 0) redn[tid / TA_WAVE] = dot;
  }
  __syncthreads();                                   // (every thread has read m_state before one writes it)
  if (!SPLIT && tid == 0) m_state[slot * H + h] = m;
  // ---- the update and the readout
  float r[VW];
#pragma unroll
  for (int e = 0; e < VW; ++e) r[e] = 0.f;
#pragma unroll
  for (int i2 = 0; i2 < ROWS; ++i2) {
    const int rw = r0 + RG * i2;
    if (on && rw < dk) {
      const float k = ks[rw], q = qs[rw];
#pragma unroll
      for (int e = 0; e < VW; ++e) {
        S[i2][e] = fmaf(keep, S[i2][e], k * v[e]);
        r[e] = fmaf(S[i2][e], q, r[e]);
      }
      float* p = st + (size_t)rw * dv + c0;
      if (VW == 4) *reinterpret_cast<float4*>(p) = float4{S[i2][0], S[i2][VW > 1 ? 1 : 0], S[i2][VW > 2 ? 2 : 0], S[i2][VW > 3 ? 3 : 0]};
      else p[0] = S[i2][0];
    }
  }
  if (on) {
#pragma unroll
    for (int e = 0; e < VW; ++e) pr[r0 * dvt + c0 + e] = r[e];
  }
  __syncthreads();
  if (SPLIT) {
    for (int j = tid; j < dvc; j += MS_NT) {
      float o = 0.f;
      for (int g = 0; g < RG; ++g) o += pr[g * dvt + j];
      o_out[((size_t)b * H + h) * dv + cb + j] = o;
    }
    return;
  }
  float below = 0.f;
#pragma unroll
  for (int w = 0; w < MS_NT / TA_WAVE; ++w) below += redn[w];
  below = 1.0f / (fmaxf(fabsf(below), expf(-m)) + MM_FLOOR_EPS);
  float ss = 0.f;
  for (int j = tid; j < dv; j += MS_NT) {            // row groups in order
    float o = 0.f;
    for (int g = 0; g < RG; ++g) o += pr[g * dv + j];
    o *= below;
    pr[j] = o;                                       // column j of row group 0 is this thread's alone now
    ss = fmaf(o, o, ss);
  }
  ss = wave_sum(ss);
  if (tid % TA_WAVE == 0) red[tid / TA_WAVE] = ss;
  __syncthreads();
  float tot = 0.f;
#pragma unroll
  for (int w = 0; w < MS_NT / TA_WAVE; ++w) tot += red[w];
  const float fac = rsqrtf(tot / (float)dv + eps);
  for (int j = tid; j < dv; j += MS_NT) {
    const float g = to_f32(row[goff + h * dv + j]);
    out[(size_t)b * H * dv + (size_t)h * dv + j] = from_f32<T>(pr[j] * fac * norm_w[h * dv + j] / (1.0f + expf(-g)));
  }
}

// What SPLIT leaves: normaliser, maximum and denominator, then norm and gate of the whole readout.
#define MF_NT 256
template <typename T>
__global__ __launch_bounds__(MF_NT) void memory_step_finish_kernel(
    const T* __restrict__ proj, int stride, int qoff, int koff, int goff, int ioff, int foff,
    const float* __restrict__ ibias, const float* __restrict__ fbias, float cap, float* __restrict__ n_state,
    float* __restrict__ m_state, const int* __restrict__ slots, int H, int dk, int dv, float qscale,
    const float* __restrict__ norm_w, float eps, const float* __restrict__ o_in, T* __restrict__ out) {
  constexpr int KEEP = 4;                            // columns a thread holds in registers; more are read twice
  __shared__ float red[MF_NT / TA_WAVE], redn[MF_NT / TA_WAVE];
  const int h = blockIdx.x, b = blockIdx.y, tid = threadIdx.x;
  const size_t at = (size_t)slots[b] * H + h;
  const T* row = proj + (size_t)b * stride;
  const float* src = o_in + ((size_t)b * H + h) * dv;
  float o[KEEP];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < KEEP; ++i) {
    const int j = tid + MF_NT * i;
    o[i] = j < dv ? src[j] : 0.f;
    ss = fmaf(o[i], o[i], ss);
  }
  for (int j = tid + MF_NT * KEEP; j < dv; j += MF_NT) ss = fmaf(src[j], src[j], ss);
  const MemoryGates gt = mm_gates(row, ioff, foff, h, ibias, fbias, cap, m_state[at]);
  float dot = 0.f;
  float* ns = n_state + at * dk;
  for (int c = tid; c < dk; c += MF_NT) {
    const float n = fmaf(gt.keep, ns[c], to_f32(row[koff + h * dk + c]) * gt.write);
    ns[c] = n;
    dot = fmaf(n, to_f32(row[qoff + h * dk + c]) * qscale, dot);
  }
  ss = wave_sum(ss);
  dot = wave_sum(dot);
  if (tid % TA_WAVE == 0) {
    red[tid / TA_WAVE] = ss;
    redn[tid / TA_WAVE] = dot;
  }
  __syncthreads();                                   // (every thread has read m_state before one writes it)
  if (tid == 0) m_state[at] = gt.m;
  float tot = 0.f, den = 0.f;
#pragma unroll
  for (int w = 0; w < MF_NT / TA_WAVE; ++w) {
    tot += red[w];
    den += redn[w];
  }
  const float below = 1.0f / (fmaxf(fabsf(den), expf(-gt.m)) + MM_FLOOR_EPS);
  const float fac = below * rsqrtf(tot * below * below / (float)dv + eps);
  auto put = [&](int j, float v) {
    const float g = to_f32(row[goff + h * dv + j]);
    out[(size_t)b * H * dv + (size_t)h * dv + j] = from_f32<T>(v * fac * norm_w[h * dv + j] / (1.0f + expf(-g)));
  };
#pragma unroll
  for (int i = 0; i < KEEP; ++i)
    if (tid + MF_NT * i < dv) put(tid + MF_NT * i, o[i]);
  for (int j = tid + MF_NT * KEEP; j < dv; j += MF_NT) put(j, src[j]);
}

static int memory_step_rows(int dk, int dv) {         // key channels a thread keeps; 0: not taken
  const int cv = dv % 4 == 0 ? dv / 4 : dv;
  if (cv < 1 || cv > MS_NT) return 0;
  const int rg = MS_NT / cv;
  const int rows = (dk + rg - 1) / rg;
  return rows <= 4 ? 4 : rows <= 8 ? 8 : rows <= 16 ? 16 : rows <= 32 ? 32 : 0;
}
static size_t memory_step_lds(int dk, int dv) {
  const int cv = dv % 4 == 0 ? dv / 4 : dv;
  return ((size_t)2 * dk + (size_t)(MS_NT / cv) * dv) * sizeof(float);
}

static bool memory_step_whole(int dk, int dv) { return memory_step_rows(dk, dv) > 0 && memory_step_lds(dk, dv) <= 60000; }
static int memory_step_tile(int dk, int dv) {         // columns of a workgroup where the head is cut; 0: not taken
  const int widest = dv % 4 == 0 ? 128 : 64;
  for (int t = widest; t >= 32; t /= 2)
    if (memory_step_rows(dk, dv % 4 == 0 ? t : t + 1) > 0 && memory_step_lds(dk, dv % 4 == 0 ? t : t + 1) <= 60000)
      return dv % 4 == 0 ? t : t + 1;                 // (an odd width: one column a thread, as where 4 does not divide dv)
  return 0;
}

// How ta_memory_step takes heads of dk x dv: 1 in one kernel, 2 in two (with scratch for the readout), 0 not at all.
extern "C" int ta_memory_step_fits(int dk, int dv) {
  if (dk < 1 || dv < 1) return 0;
  if (memory_step_whole(dk, dv)) return 1;
  const int t = memory_step_tile(dk, dv);
  return t > 0 && (dv + t - 1) / t <= 65535 ? 2 : 0;
}

// proj: [batch] rows, stride apart, with q and k (H*dk each), v and the output gate (H*dv each), the input and
// the forget gates' numbers (H each) at columns qoff, koff, voff, goff, ioff, foff. state [slots, H, dk, dv],
// n_state [slots, H, dk], m_state [slots, H] float32; norm_w [H*dv]; out [batch, H*dv] = the readout over its
// root mean square per head, times norm_w, times sigmoid(gate). scratch: [batch, H, dv] float32 where
// ta_memory_step_fits says 2 (else null).
extern "C" int ta_memory_step(hipStream_t stream, int dtype, const void* proj, int stride, int qoff, int koff, int voff,
                              int goff, int ioff, int foff, const float* ibias, const float* fbias, float cap,
                              float* state, float* n_state, float* m_state, const int* slots, int batch, int H, int dk,
                              int dv, float qscale, const float* norm_w, float eps, float* scratch, void* out) {
  TA_REQUIRE(batch > 0 && batch <= 65535 && H >= 1 && H <= 65535, "ta_memory_step: batch %d, %d heads", batch, H);
  TA_REQUIRE(ta_memory_step_fits(dk, dv), "ta_memory_step: heads of %d x %d", dk, dv);
  TA_REQUIRE(qoff >= 0 && koff >= 0 && voff >= 0 && goff >= 0 && ioff >= 0 && foff >= 0 && stride >= qoff + H * dk &&
             stride >= koff + H * dk && stride >= voff + H * dv && stride >= goff + H * dv && stride >= ioff + H &&
             stride >= foff + H, "ta_memory_step: rows of %d are too short", stride);
  TA_REQUIRE(cap > 0.f, "ta_memory_step: the cap must be positive, got %g", (double)cap);
  TA_REQUIRE(dv % 4 != 0 || (uintptr_t)state % 16 == 0, "ta_memory_step: the state must be 16-byte aligned");
  const bool split = !memory_step_whole(dk, dv);
  TA_REQUIRE(!split || scratch != nullptr, "ta_memory_step: heads of %d x %d need scratch memory", dk, dv);
  TA_REQUIRE(dtype == TA_F32 || dtype == TA_BF16, "ta_memory_step: unknown dtype %d", dtype);
  const int dvt = split ? memory_step_tile(dk, dv) : dv;
  const int rows = memory_step_rows(dk, dvt);
  const size_t lds = memory_step_lds(dk, dvt);
  dim3 g(H, batch, split ? (dv + dvt - 1) / dvt : 1);
#define MS_KERNEL(T, VWV, RW, SP)                                                                                   \
  memory_step_kernel<T, VWV, RW, SP><<<g, MS_NT, lds, stream>>>(                                                    \
      (const T*)proj, stride, qoff, koff, voff, goff, ioff, foff, ibias, fbias, cap, state, n_state, m_state, slots, \
      H, dk, dv, qscale, norm_w, eps, (T*)out, dvt, scratch)
#define MS_RUN(T, VWV, RW) \
  if (split) MS_KERNEL(T, VWV, RW, true); else MS_KERNEL(T, VWV, RW, false)
#define MS_BY_ROWS(T, VWV)                 \
  switch (rows) {                          \
    case 4: MS_RUN(T, VWV, 4); break;      \
    case 8: MS_RUN(T, VWV, 8); break;      \
    case 16: MS_RUN(T, VWV, 16); break;    \
    default: MS_RUN(T, VWV, 32); break;    \
  }
#define MS_BY_COLS(T) \
  if (dv % 4 == 0) { MS_BY_ROWS(T, 4) } else { MS_BY_ROWS(T, 1) }
  if (dtype == TA_F32) { MS_BY_COLS(float) } else { MS_BY_COLS(bf16_t) }
#undef MS_BY_COLS
#undef MS_BY_ROWS
#undef MS_RUN
#undef MS_KERNEL
  const int rc = ta_check_launch("ta_memory_step");
  if (rc != 0 || !split) return rc;
#define MF_RUN(T)                                                                                                   \
  memory_step_finish_kernel<T><<<dim3(H, batch), MF_NT, 0, stream>>>((const T*)proj, stride, qoff, koff, goff, ioff, \
                                                                     foff, ibias, fbias, cap, n_state, m_state, slots, \
                                                                     H, dk, dv, qscale, norm_w, eps, scratch, (T*)out)
  if (dtype == TA_F32) MF_RUN(float); else MF_RUN(bf16_t);
#undef MF_RUN
  return ta_check_launch("ta_memory_step");
}
