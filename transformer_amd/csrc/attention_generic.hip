// Causal grouped-query attention over the paged cache, float32 arithmetic on the
// vector ALU, for any key width and any value width up to 256 (the two may differ)
// and both storage types. It serves prompts and single tokens alike.
//
// A workgroup owns 16 "rows" of one (sequence, kv head): row = (query token,
// query head inside the kv head's group), so the heads of a group share every
// key/value load. Keys are walked in chunks of 32 aligned to absolute positions
// and every row's running maximum, sum and output are updated in that order, so
// a row's result depends only on its own query and keys: not on the batch, not
// on how the tokens were cut into steps, not on which pages hold the keys.
//
// Options (all off in the plain entry points): scores capped by cap * tanh(score / cap); one more
// term in the softmax denominator that has no value (a "sink": exp(0), or exp of a learned number
// per head); the result multiplied by the sigmoid of a gate, element by element or one number per head;
// a window that besides the last keys also shows a sequence's first `keep` keys.
#include "common.h"

#define ROWS 16
#define CHUNK 32

__device__ __forceinline__ float group16_max(float v) {
#pragma unroll
  for (int o = 8; o > 0; o >>= 1) v = fmaxf(v, __shfl_xor(v, o, 16));
  return v;
}
__device__ __forceinline__ float group16_sum(float v) {
#pragma unroll
  for (int o = 8; o > 0; o >>= 1) v += __shfl_xor(v, o, 16);
  return v;
}

template <typename T>
__global__ __launch_bounds__(256) void attn_generic_kernel(
    const T* __restrict__ q, int q_stride, T* __restrict__ out, int out_stride,
    const T* __restrict__ kcache, const T* __restrict__ vcache,
    const int* __restrict__ block_table, int max_blocks, const int* __restrict__ cu_q,
    const int* __restrict__ pos0, int nh, int nkv, int dh, int dv, float scale, int window,
    float softcap, int sink_mode, const float* __restrict__ sink, const T* __restrict__ gate, int gate_stride,
    int gate_dv, int keep, int chunk) {
  extern __shared__ float smem[];
  const int group = nh / nkv;
  const int b = blockIdx.z, kvh = blockIdx.y;
  const int q0 = cu_q[b], qlen = cu_q[b + 1] - q0;
  const int nrows = qlen * group;
  const int row0 = blockIdx.x * ROWS;
  if (row0 >= nrows) return;
  const int p0 = pos0[b];
  const int rloc = threadIdx.x / 16, lane = threadIdx.x % 16;
  const int row = row0 + rloc;
  const bool row_ok = row < nrows;
  const int qi = row_ok ? row / group : 0;
  const int head = kvh * group + (row_ok ? row % group : 0);
  const int DHP = (dh > dv ? dh : dv) + 1;
  float* Qs = smem;                 // [ROWS][dh]
  float* KVs = Qs + ROWS * dh;      // [CHUNK][dh + 1]
  float* Ps = KVs + CHUNK * DHP;    // [ROWS][CHUNK]

  for (int i = threadIdx.x; i < ROWS * dh; i += 256) {
    const int r = i / dh, d = i - r * dh, rr = row0 + r;
    float v = 0.f;
    if (rr < nrows)
      v = to_f32(q[(size_t)(q0 + rr / group) * q_stride + (size_t)(kvh * group + rr % group) * dh + d]);
    Qs[i] = v;
  }

  // key range of this tile of rows
  const int qi_min = row0 / group;
  const int last_row = (row0 + ROWS - 1 < nrows - 1) ? row0 + ROWS - 1 : nrows - 1;
  const int tile_end = p0 + last_row / group + 1;                       // exclusive
  const int tile_start = ta_first_key(p0 + qi_min + 1, window, chunk);
  const int my_end = p0 + qi + 1;
  const int my_start = ta_first_key(my_end, window, chunk);

  const int nd = (dv + 15) / 16;          // output columns lane, lane + 16, ... of this lane
  float acc[16];
#pragma unroll
  for (int i = 0; i < 16; ++i) acc[i] = 0.f;
  float m = -INFINITY, l = 0.f;

  const int* table = block_table + (size_t)b * max_blocks;
  // chunks of the kept first keys that the window has left behind, then the window's
  const int win_chunk = tile_start / CHUNK;
  int c = keep > 0 ? 0 : win_chunk;
  for (; c * CHUNK < tile_end; ++c) {
    const int key0 = c * CHUNK;
    if (c < win_chunk && key0 >= keep) {       // nothing between the kept keys and the window is read
      c = win_chunk - 1;
      continue;
    }
    const size_t page = (size_t)table[key0 / TA_PAGE];
    const size_t base = ((page * nkv + kvh) * TA_PAGE + key0 % TA_PAGE) * (size_t)dh;
    const size_t vbase = (page * nkv + kvh) * (size_t)dv * TA_PAGE + key0 % TA_PAGE;
    // ---- K chunk -> LDS (keys that are not written yet read as zero)
    for (int i = threadIdx.x; i < CHUNK * dh; i += 256) {
      const int k = i / dh, d = i - k * dh;
      KVs[k * DHP + d] = (key0 + k < tile_end) ? to_f32(kcache[base + i]) : 0.f;
    }
    __syncthreads();
    float s0 = 0.f, s1 = 0.f;
    {
      const float* qr = Qs + rloc * dh;
      const float* k0 = KVs + lane * DHP;
      const float* k1 = KVs + (lane + 16) * DHP;
      for (int d = 0; d < dh; ++d) {
        const float qv = qr[d];
        s0 = fmaf(qv, k0[d], s0);
        s1 = fmaf(qv, k1[d], s1);
      }
    }
    const int kk0 = key0 + lane, kk1 = kk0 + 16;
    const bool v0 = row_ok && (kk0 >= my_start || kk0 < keep) && kk0 < my_end;
    const bool v1 = row_ok && (kk1 >= my_start || kk1 < keep) && kk1 < my_end;
    s0 *= scale;
    s1 *= scale;
    if (softcap > 0.f) {              // capped scores: cap * tanh(score / cap)
      s0 = softcap * tanhf(s0 / softcap);
      s1 = softcap * tanhf(s1 / softcap);
    }
    s0 = v0 ? s0 : -INFINITY;
    s1 = v1 ? s1 : -INFINITY;
    const float m_new = fmaxf(m, group16_max(fmaxf(s0, s1)));
    float alpha = 1.f, e0 = 0.f, e1 = 0.f;
    if (m_new != -INFINITY) {
      alpha = expf(m - m_new);          // m = -inf gives 0
      e0 = v0 ? expf(s0 - m_new) : 0.f;
      e1 = v1 ? expf(s1 - m_new) : 0.f;
    }
    l = l * alpha + group16_sum(e0 + e1);
    m = m_new;
#pragma unroll
    for (int i = 0; i < 16; ++i) acc[i] *= alpha;
    Ps[rloc * CHUNK + lane] = e0;
    Ps[rloc * CHUNK + lane + 16] = e1;
    __syncthreads();
    // ---- V chunk -> LDS
    for (int i = threadIdx.x; i < CHUNK * dv; i += 256) {     // value pages are [dv][TA_PAGE]
      const int d = i / CHUNK, k = i - d * CHUNK;
      KVs[k * DHP + d] = (key0 + k < tile_end) ? to_f32(vcache[vbase + (size_t)d * TA_PAGE + k]) : 0.f;
    }
    __syncthreads();
    {
      const float* pr = Ps + rloc * CHUNK;
      for (int k = 0; k < CHUNK; ++k) {
        const float p = pr[k];
        const float* vr = KVs + k * DHP + lane;
#pragma unroll
        for (int i = 0; i < 16; ++i)
          if (i < nd && 16 * i + lane < dv) acc[i] = fmaf(p, vr[16 * i], acc[i]);
      }
    }
    __syncthreads();
  }
  if (row_ok) {
    // a sink is one more term of the denominator with a score of its own and no value:
    // sink_mode 1: score 0 for every head; 2: sink[head]
    if (sink_mode != 0) {
      const float sv = sink_mode == 2 ? sink[head] : 0.f;
      const float m_new = fmaxf(m, sv);
      const float alpha = expf(m - m_new);          // m = -inf (no key seen) gives 0
      l = l * alpha + expf(sv - m_new);
#pragma unroll
      for (int i = 0; i < 16; ++i) acc[i] *= alpha;
    }
    float inv = l > 0.f ? 1.0f / l : 0.f;
    if (gate && gate_dv == 0)          // one number per head
      inv *= 1.0f / (1.0f + expf(-to_f32(gate[(size_t)(q0 + qi) * gate_stride + head])));
    T* o = out + (size_t)(q0 + qi) * out_stride + (size_t)head * dv + lane;
    // the gate's rows hold gate_dv columns per head (the values' own width where the cache pads them)
    const T* gt = gate && gate_dv > 0 ? gate + (size_t)(q0 + qi) * gate_stride + (size_t)head * gate_dv + lane : nullptr;
#pragma unroll
    for (int i = 0; i < 16; ++i)
      if (i < nd && 16 * i + lane < dv) {
        float r = acc[i] * inv;
        if (gt && 16 * i + lane < gate_dv) r *= 1.0f / (1.0f + expf(-to_f32(gt[16 * i])));      // the heads' sigmoid gate
        o[16 * i] = from_f32<T>(r);
      }
  }
}

// q: [nt, ...] with q_stride elements between tokens, head h at offset h*dh.
// out: [nt, nh*dv] with out_stride elements between tokens.
// kcache: one layer, [pages][nkv][TA_PAGE][dh]; vcache: [pages][nkv][dv][TA_PAGE].
// block_table: [B][max_blocks].
// cu_q: [B+1] first token of each sequence in q. pos0: [B] tokens cached before this
// step (the step's own keys are already in the cache). window <= 0: all keys.
static int attention_generic_launch(hipStream_t stream, int dtype, const void* q, int q_stride,
                                    void* out, int out_stride, const void* kcache,
                                    const void* vcache, const int* block_table, int max_blocks,
                                    const int* cu_q, const int* pos0, int batch, int max_qlen,
                                    int nh, int nkv, int dh, int dv, float scale, int window,
                                    float softcap = 0.f, int sink_mode = 0, const float* sink = nullptr,
                                    const void* gate = nullptr, int gate_stride = 0, int gate_dv = 0, int keep = 0,
                                    int chunk = 0) {
  TA_REQUIRE(batch >= 0 && max_qlen >= 0, "ta_attention_generic: bad batch=%d max_qlen=%d", batch, max_qlen);
  TA_REQUIRE(sink_mode >= 0 && sink_mode <= 2 && (sink_mode != 2 || sink != nullptr) && softcap >= 0.f,
             "ta_attention_generic: sink mode %d, cap %f", sink_mode, softcap);
  TA_REQUIRE(gate == nullptr || (gate_dv >= 0 && gate_dv <= dv && gate_stride >= nh * (gate_dv > 0 ? gate_dv : 1)),
             "ta_attention_generic: gate rows of %d", gate_stride);
  TA_REQUIRE(keep >= 0 && (keep == 0 || window > 0), "ta_attention_generic: %d kept keys beside a window of %d", keep, window);
  TA_REQUIRE(chunk >= 0 && (chunk == 0 || window <= 0), "ta_attention_generic: chunks of %d beside a window of %d", chunk, window);
  TA_REQUIRE(nh > 0 && nkv > 0 && nh % nkv == 0, "ta_attention_generic: %d heads do not divide into %d kv heads", nh, nkv);
  TA_REQUIRE(dh >= 1 && dh <= 256 && dv >= 1 && dv <= 256,
             "ta_attention_generic: key width %d / value width %d outside [1, 256]", dh, dv);
  TA_REQUIRE(q_stride >= nh * dh && out_stride >= nh * dv, "ta_attention_generic: strides too small");
  TA_REQUIRE(max_blocks > 0, "ta_attention_generic: empty block table");
  TA_REQUIRE(batch <= 65535 && nkv <= 65535, "ta_attention_generic: grid too large");
  if (batch == 0 || max_qlen == 0) return 0;
  const int group = nh / nkv;
  dim3 g((max_qlen * group + ROWS - 1) / ROWS, nkv, batch), blk(256);
  const size_t lds = (size_t)(ROWS * dh + CHUNK * ((dh > dv ? dh : dv) + 1) + ROWS * CHUNK) * sizeof(float);
  if (dtype == TA_F32)
    attn_generic_kernel<float><<<g, blk, lds, stream>>>(
        (const float*)q, q_stride, (float*)out, out_stride, (const float*)kcache,
        (const float*)vcache, block_table, max_blocks, cu_q, pos0, nh, nkv, dh, dv, scale, window,
        softcap, sink_mode, sink, (const float*)gate, gate_stride, gate_dv, keep, chunk);
  else if (dtype == TA_BF16)
    attn_generic_kernel<bf16_t><<<g, blk, lds, stream>>>(
        (const bf16_t*)q, q_stride, (bf16_t*)out, out_stride, (const bf16_t*)kcache,
        (const bf16_t*)vcache, block_table, max_blocks, cu_q, pos0, nh, nkv, dh, dv, scale, window,
        softcap, sink_mode, sink, (const bf16_t*)gate, gate_stride, gate_dv, keep, chunk);
  else
    return ta_fail("ta_attention_generic: unknown dtype %d", dtype);
  return ta_check_launch("ta_attention_generic");
}

extern "C" int ta_attention_generic(hipStream_t stream, int dtype, const void* q, int q_stride,
                                    void* out, int out_stride, const void* kcache,
                                    const void* vcache, const int* block_table, int max_blocks,
                                    const int* cu_q, const int* pos0, int batch, int max_qlen,
                                    int nh, int nkv, int dh, float scale, int window) {
  return attention_generic_launch(stream, dtype, q, q_stride, out, out_stride, kcache, vcache, block_table,
                                  max_blocks, cu_q, pos0, batch, max_qlen, nh, nkv, dh, dh, scale, window);
}

// The same with values of another width than the keys: dv columns per head in vcache and out.
extern "C" int ta_attention_generic_dv(hipStream_t stream, int dtype, const void* q, int q_stride,
                                       void* out, int out_stride, const void* kcache,
                                       const void* vcache, const int* block_table, int max_blocks,
                                       const int* cu_q, const int* pos0, int batch, int max_qlen,
                                       int nh, int nkv, int dh, int dv, float scale, int window) {
  return attention_generic_launch(stream, dtype, q, q_stride, out, out_stride, kcache, vcache, block_table,
                                  max_blocks, cu_q, pos0, batch, max_qlen, nh, nkv, dh, dv, scale, window);
}

// The same with the options of a capped, sunk and gated softmax: softcap > 0: score <- softcap *
// tanh(score / softcap) after the scale; sink_mode 1: the denominator holds one more term exp(0);
// 2: exp(sink[head]) (float32 [nh]); gate: rows [nt, >= nh*gate_dv] whose sigmoid multiplies the first gate_dv
// columns of every head of the result (gate_dv <= dv; 0: rows [nt, >= nh] with one number per head). keep:
// with a window, the first `keep` keys of a sequence are seen as well. chunk > 0 (without a window): a query
// at position p sees the keys from (p / chunk) * chunk on.
extern "C" int ta_attention_generic_sink(hipStream_t stream, int dtype, const void* q, int q_stride,
                                         void* out, int out_stride, const void* kcache,
                                         const void* vcache, const int* block_table, int max_blocks,
                                         const int* cu_q, const int* pos0, int batch, int max_qlen,
                                         int nh, int nkv, int dh, int dv, float scale, int window,
                                         float softcap, int sink_mode, const float* sink, const void* gate,
                                         int gate_stride, int gate_dv, int keep, int chunk) {
  return attention_generic_launch(stream, dtype, q, q_stride, out, out_stride, kcache, vcache, block_table,
                                  max_blocks, cu_q, pos0, batch, max_qlen, nh, nkv, dh, dv, scale, window,
                                  softcap, sink_mode, sink, gate, gate_stride, gate_dv, keep, chunk);
}
