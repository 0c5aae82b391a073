// Shared device helpers and the host-side error channel of the kernel library (gfx950, wave64).
#pragma once
#include <hip/hip_runtime.h>
#include <stdint.h>
#include <stdio.h>
#include <stdarg.h>

typedef uint16_t bf16_t;   // raw bfloat16 bits

enum { TP_F32 = 0, TP_BF16 = 1 };

// ---- host: errors -----------------------------------------------------------------------------
// Every entry point returns 0, or a non-zero code after storing a message that tp_last_error() gives back.
extern "C" const char* tp_last_error();
int tp_fail(const char* fmt, ...);
int tp_check_launch(const char* what);

#define TP_REQUIRE(cond, ...) do { if (!(cond)) return tp_fail(__VA_ARGS__); } while (0)

static inline int tp_cdiv(long a, long b) { return (int)((a + b - 1) / b); }

// ---- device: number formats ------------------------------------------------------------------
__device__ __forceinline__ float bf16_to_f32(bf16_t v) { return __uint_as_float(((uint32_t)v) << 16); }

__device__ __forceinline__ bf16_t f32_to_bf16(float f) {      // round to nearest even; NaN stays NaN
    uint32_t u = __float_as_uint(f);
    if ((u & 0x7fffffffu) > 0x7f800000u) return (bf16_t)((u >> 16) | 0x40);
    u += 0x7fffu + ((u >> 16) & 1u);
    return (bf16_t)(u >> 16);
}

__device__ __forceinline__ float ld_f32(const float* p) { return *p; }
__device__ __forceinline__ float ld_f32(const bf16_t* p) { return bf16_to_f32(*p); }
__device__ __forceinline__ void st_f32(float* p, float v) { *p = v; }
__device__ __forceinline__ void st_f32(bf16_t* p, float v) { *p = f32_to_bf16(v); }

// ---- device: reductions over a wave of 64 and over a block -------------------------------------
__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) v += __shfl_xor(v, o, 64);
    return v;
}
__device__ __forceinline__ float wave_max(float v) {
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) v = fmaxf(v, __shfl_xor(v, o, 64));
    return v;
}

// Sum over a block of up to 1024 threads; every thread gets the result.  `red` holds 16 floats of LDS.
// The order of additions depends only on the block size, never on timing.
__device__ __forceinline__ float block_sum(float v, float* red) {
    v = wave_sum(v);
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, nw = (blockDim.x + 63) >> 6;
    __syncthreads();                       // red may still be read from an earlier call
    if (lane == 0) red[wave] = v;
    __syncthreads();
    float t = 0.f;
    for (int i = 0; i < nw; i++) t += red[i];
    return t;
}

// The same where `red` has not been used by the block before (a call's own 16 floats): one barrier less.
__device__ __forceinline__ float block_sum_once(float v, float* red) {
    v = wave_sum(v);
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, nw = (blockDim.x + 63) >> 6;
    if (lane == 0) red[wave] = v;
    __syncthreads();
    float t = 0.f;
    for (int i = 0; i < nw; i++) t += red[i];
    return t;
}

// ---- device: functions of the model ---------------------------------------------------------------
__device__ __forceinline__ float gelu_tanh_f(float g) {
    return 0.5f * g * (1.0f + tanhf(0.7978845608f * (g + 0.044715f * g * g * g)));
}
__device__ __forceinline__ float softcap_f(float s, float cap) { return cap * tanhf(s / cap); }
// The same function for the bf16 products' epilogues, where it is evaluated once per output element of the largest
// product: 0.5 g (1 + tanh u) = g / (1 + e^(-2u)), one exponential and one reciprocal instruction instead of the
// library's tanh (relative error of a few 1e-7; the result is rounded to bf16).
__device__ __forceinline__ float gelu_tanh_fast(float g) {
    constexpr float C1 = -2.f * 0.7978845608f * 1.4426950408889634f, C3 = C1 * 0.044715f;
    return g * __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(g * __builtin_fmaf(C3, g * g, C1)));
}

// ---- attention whose scores and outputs depend on positions and gates ------------------------------------------------------
// Handed to the attention kernels by pointer (null: none of it).  The scores of the query at position p are multiplied by
// 1 + temp_coef ln(floor((p + 1) / temp_every) + 1) (temp_every 0: not at all); after the cap, head h's score on the key at
// distance n gets bias[h][min(n, reach)] added; head h's output of row r is multiplied by sigmoid(gate[r][h]), gate being
// rows of either dtype, float32 ones possibly in K slices of a product that are added in slice order.
struct TpPositional {
    const float* bias; long reach;
    const void* gate; long gate_f32, gate_slices, gate_slice_stride, gate_stride;
    float temp_coef; int temp_every;
};
__device__ __forceinline__ float query_temperature(const TpPositional& s, int p) {
    return s.temp_every > 0 ? 1.f + s.temp_coef * logf((float)((p + 1) / s.temp_every + 1)) : 1.f;
}
__device__ __forceinline__ float head_gate(const TpPositional& s, size_t row, int h) {
    const size_t at = row * s.gate_stride + h;
    float g = 0.f;
    if (s.gate_f32) for (int i = 0; i < (int)s.gate_slices; i++) g += ((const float*)s.gate)[i * s.gate_slice_stride + at];
    else g = bf16_to_f32(((const bf16_t*)s.gate)[at]);
    return 1.f / (1.f + expf(-g));
}
static inline bool tp_positional_ok(const TpPositional* s) {
    return !s || ((!s->bias || s->reach >= 0) && s->temp_every >= 0 && (!s->gate || (s->gate_slices >= 1 && (s->gate_f32 || s->gate_slices == 1))));
}

// ---- gate activations of a gated product -----------------------------------------------------------------------
// The activations offered are of one form, act(g) = g / (1 + 2^(g (c1 + c3 g^2))): gelu-tanh (above) with
// c1 = -2 * 0.7978845608 * log2(e), c3 = c1 * 0.044715, and SiLU, g / (1 + e^-g), with c1 = -log2(e), c3 = 0.  The
// bf16 products' epilogues take the two constants (`epi.x`, `epi.y`) and have no branch on the activation's kind.
// ReLU is the limit of the form for c1 -> -infinity: with c1 = -1e30 the power of two is 0 for every g above 1e-28
// and infinite for every g below -1e-28, so the quotient is g or -0 (and within 1e-28 of 0 in between).
// A fourth, g sigmoid(1.702 g), is SiLU's form with c1 = -1.702 log2(e).  A gated product may also cut its sums first:
// g' = min(g, limit), u' = clamp(u, -limit, limit), out = act(g') (u' + shift); limit = infinity and shift = 0 leave
// the plain product act(g) u, bit for bit (`epi.z`, `epi.w`).
enum { TP_ACT_GELU_TANH = 0, TP_ACT_SILU = 1, TP_ACT_RELU = 2, TP_ACT_QUICK_GELU = 3 };
// which elements of a head a rotation pairs: (f, f + rotary_dim / 2) as the reference does
// (runtime/cuda/codebook_gemv.cu:219-230), or neighbours (2f, 2f + 1)
enum { TP_ROPE_HALVES = 0, TP_ROPE_NEIGHBOURS = 1 };
static inline bool tp_gate_constants(int act, float* c1, float* c3) {
    constexpr float LOG2E = 1.4426950408889634f;
    if (act == TP_ACT_GELU_TANH) { *c1 = -2.f * 0.7978845608f * LOG2E; *c3 = *c1 * 0.044715f; return true; }
    if (act == TP_ACT_SILU) { *c1 = -LOG2E; *c3 = 0.f; return true; }
    if (act == TP_ACT_RELU) { *c1 = -1e30f; *c3 = 0.f; return true; }
    if (act == TP_ACT_QUICK_GELU) { *c1 = -1.702f * LOG2E; *c3 = 0.f; return true; }
    return false;
}
__device__ __forceinline__ float gate_act_fast(float g, float4 epi) {
    return g * __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(g * __builtin_fmaf(epi.y, g * g, epi.x)));
}
// a gated product's output element from its gate and up sums
__device__ __forceinline__ float gated_unit_fast(float g, float u, float4 epi) {
    g = fminf(g, epi.z);
    u = fminf(fmaxf(u, -epi.z), epi.z);
    return gate_act_fast(g, epi) * (u + epi.w);
}
// the same in full float32 arithmetic, for the float32 path
__device__ __forceinline__ float gate_act_exact(float g, int act) {
    if (act == TP_ACT_QUICK_GELU) return g / (1.f + expf(-1.702f * g));
    return act == TP_ACT_SILU ? g / (1.f + expf(-g)) : (act == TP_ACT_RELU ? fmaxf(g, 0.f) : gelu_tanh_f(g));
}
__device__ __forceinline__ float gated_unit_exact(float g, float u, int act, float limit, float shift) {
    g = fminf(g, limit);
    u = fminf(fmaxf(u, -limit), limit);
    return gate_act_exact(g, act) * (u + shift);
}
