// Shared device helpers and the host-side error convention of the kernel library.
//
// Every exported function returns 0 on success. On failure it returns non-zero
// and leaves a message that ta_last_error() returns; arguments are checked on
// the host before any kernel is launched, so a refused call has launched nothing.
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>
#include <stdio.h>
#include <stdarg.h>

#define TA_WAVE 64
#define TA_PAGE 64   // tokens per cache page; the Python side asserts the same number
#define TA_UNIT_INTS 8    // int32 values in the record of a unit of work of the single-token attention
#define TA_MAX_PLANES 8   // parts in which a product may leave a float32 result for the next norm to add

enum ta_dtype { TA_F32 = 0, TA_BF16 = 1 };

struct bf16_t {
  uint16_t v;
};

__device__ __forceinline__ float to_f32(float x) { return x; }
__device__ __forceinline__ float to_f32(bf16_t x) { return __uint_as_float(((uint32_t)x.v) << 16); }

// round to nearest even with the hardware's conversion (v_cvt_pk_bf16_f32 on gfx950)
__device__ __forceinline__ uint16_t f32_to_bf16_bits(float f) {
  const __bf16 b = (__bf16)f;
  return __builtin_bit_cast(uint16_t, b);
}
// two values in one instruction: a in the low half, b in the high half
__device__ __forceinline__ uint32_t f32x2_to_bf16x2_bits(float a, float b) {
  typedef __attribute__((__vector_size__(2 * sizeof(__bf16)))) __bf16 bf16x2_t;
  bf16x2_t v;
  v[0] = (__bf16)a;
  v[1] = (__bf16)b;
  return __builtin_bit_cast(uint32_t, v);
}

template <typename T> __device__ __forceinline__ T from_f32(float f);
template <> __device__ __forceinline__ float from_f32<float>(float f) { return f; }
template <> __device__ __forceinline__ bf16_t from_f32<bf16_t>(float f) {
  bf16_t r;
  r.v = f32_to_bf16_bits(f);
  return r;
}

// How a product that owns a gate column and an up column joins them: silu(gate) * up, or, with a
// limit, g * sigmoid(slope * g) * (u + shift) with g = min(gate, limit), u = clamp(up, -limit, limit).
struct TaGlu {
  float limit, slope, shift;      // limit 0: silu
};
__device__ __forceinline__ float ta_glu(const TaGlu& p, float g, float u) {
  if (p.limit > 0.f) {
    g = fminf(g, p.limit);
    u = fminf(fmaxf(u, -p.limit), p.limit);
    return g / (1.0f + expf(-p.slope * g)) * (u + p.shift);
  }
  return g / (1.0f + expf(-g)) * u;
}

// The first key that a query sees whose own key is the last before `end`: a window shows the last
// `window` keys, chunks those from its chunk's start on (chunk counted from position 0); both 0: all.
__device__ __forceinline__ int ta_first_key(int end, int window, int chunk) {
  if (chunk > 0) return end > 0 ? (int)((unsigned)(end - 1) / (unsigned)chunk * (unsigned)chunk) : 0;
  return (window > 0 && end > window) ? end - window : 0;
}

__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
  for (int o = TA_WAVE / 2; o > 0; o >>= 1) v += __shfl_xor(v, o, TA_WAVE);
  return v;
}
__device__ __forceinline__ float wave_max(float v) {
#pragma unroll
  for (int o = TA_WAVE / 2; o > 0; o >>= 1) v = fmaxf(v, __shfl_xor(v, o, TA_WAVE));
  return v;
}

// Sums over 16, 32 or 64 neighbouring lanes that leave the same bits in each of them.
template <int CTRL>
__device__ __forceinline__ float ta_dpp(float x) {
  return __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(x), CTRL, 0xf, 0xf, true));
}
__device__ __forceinline__ float ta_sum16(float x) {       // pairs, quads, halves of a row, rows
  x += ta_dpp<0xB1>(x);      // lanes 1 apart
  x += ta_dpp<0x4E>(x);      // 2 apart
  x += ta_dpp<0x141>(x);     // mirrored in eights
  x += ta_dpp<0x140>(x);     // mirrored in sixteens
  return x;
}
// two sums at once
template <int LANES>
__device__ __forceinline__ void ta_sums2(float& w, float& r) {
  static_assert(LANES == 16 || LANES == 32 || LANES == 64, "lanes that share a sum");
  if (LANES == 16) {
    w = ta_sum16(w);
    r = ta_sum16(r);
    return;
  }
  // rows of 16 lanes trade places: the even ones are left with what both rows have of w, the odd ones with
  // theirs of r, one exchange sums either, and a second trade hands both to all lanes
  const auto a = __builtin_amdgcn_permlane16_swap(__float_as_uint(w), __float_as_uint(r), false, false);
  float t = ta_sum16(__uint_as_float(a[0]) + __uint_as_float(a[1]));
  if (LANES == 64) {
    const auto h = __builtin_amdgcn_permlane32_swap(__float_as_uint(t), __float_as_uint(t), false, false);
    t = __uint_as_float(h[0]) + __uint_as_float(h[1]);
  }
  const auto c = __builtin_amdgcn_permlane16_swap(__float_as_uint(t), __float_as_uint(t), false, false);
  w = __uint_as_float(c[0]);
  r = __uint_as_float(c[1]);
}

// ---------------------------------------------------------------- host side
int ta_fail(const char* fmt, ...);            // records the message, returns 1
int ta_check_launch(const char* what);        // hipGetLastError -> message

#define TA_REQUIRE(cond, ...)            \
  do {                                   \
    if (!(cond)) return ta_fail(__VA_ARGS__); \
  } while (0)
