// The gated delta rule: a matrix per head that decays, forgets along the key it is about to write, and is read at once.
//
//   per head, for a token with key k and query q (unit vectors, q also times dk^(-1/2)), value v, decay g and step beta:
//   S <- g S;   u = beta (v - S^T k);   S <- S + k u^T;   o = S^T q
//   g = exp(-exp(a_log) softplus(a + dt_bias)),  beta = sigmoid(b);  x / sqrt(sum x^2 + 1e-6) makes a unit vector
//
// S, the decays and steps, the norms of q and k and every sum are float32.  q, k and v arrive as the short convolutions
// left them (bfloat16 in a bfloat16 engine); heads share the queries and keys of head h / (H / G).  A column of S (one value
// element) goes on by itself, so the value columns are what is spread over waves and blocks.
//
// Two forms.  `delta_rows_k` takes a sequence's tokens one by one: 16 columns a wave, its 64 lanes holding 4 columns by
// a sixteenth of the rows each (a decode step, short portions, float32 engines).  Long bfloat16 steps run in chunks of 64
// tokens on the matrix cores.  With G_t the sum of log decays up to t inside a chunk, S_0 the state it starts from,
//   (I + L) U = diag(beta) (V - diag(e^G) K S_0),        L_ts = beta_t e^(G_t - G_s) (k_t . k_s) for s < t
//   O = diag(e^G) Q S_0 + A U,                           A_ts = e^(G_t - G_s) (q_t . k_s) for s <= t
//   S_C = e^(G_C) S_0 + (diag(e^(G_C - G)) K)^T U
// What does not depend on S_0 (the inverse of I + L, A, the scalars of every token, K transposed) is formed for all chunks
// at once by `delta_prepare_k`; `delta_chunks_k` then walks a sequence's chunks in order.  No exponent is ever positive.
// Products with a float32 operand stay exact to 24 bits: the operand is split into three bfloat16 terms (a bfloat16
// operand, k or q, is one term), whose products the matrix cores add up in float32.
#include "common.h"

typedef __attribute__((__vector_size__(8 * sizeof(__bf16)))) __bf16 dl_bf16x8;
typedef __attribute__((__vector_size__(4 * sizeof(float)))) float dl_f32x4;

struct DeltaArgs {
    const void* q; long q_stride; const void* k; long k_stride; const void* v; long v_stride;
    const void* b; const void* a; long gate_stride;      // [M, H] each, of the rows' dtype
    const float* a_log; const float* dt_bias;            // [H]
    float* state;                                        // [slots, H, dk, dv]
    const int* slot_ids; const int* cu_rows; float* y;   // y [M, H dv]
    int n_seq, H, G, dk, dv; float q_scale;
    // chunks: for (sequence, chunk) c and head h, at (c H + h): T' and A in three terms of [64][64], four rows of 64 scalars
    // (e^G / |k|, q_scale e^G / |q|, e^(G_C - G) / |k|, e^(G_C)); for kv head j, at (c G + j): K transposed [dkp][64]
    int n_chunks, dkp; bf16_t* ws_mat; float* ws_scal; bf16_t* ws_kt;
};

namespace {
constexpr int DC = 64;                           // tokens of a chunk
constexpr int DCP = DC + 8;                      // a row of 64 terms in LDS
constexpr float UNIT_EPS = 1e-6f;

__device__ __forceinline__ float log_decay_of(float a, float dt_bias, float a_log) {
    const float z = a + dt_bias;
    return -expf(a_log) * (fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))));
}
__device__ __forceinline__ float step_of(float b) { return 1.f / (1.f + expf(-b)); }
__device__ __forceinline__ float rows_sum(float v) {      // over the 16 groups of rows (lanes 4 apart)
#pragma unroll
    for (int o = 4; o < 64; o <<= 1) v += __shfl_xor(v, o, 64);
    return v;
}
template <typename T> struct alignas(sizeof(T) * 4) Quad { T v[4]; };

// R elements of a row from row0 on, zeros from `rows` on; VEC: rows and everything else in whole quads
template <typename T, int R, bool VEC>
__device__ __forceinline__ void load_part(float (&dst)[R], const T* p, int row0, int rows) {
    if constexpr (VEC) {
#pragma unroll
        for (int i = 0; i < R; i += 4) {
            const bool ok = row0 + i < rows;
            const Quad<T> t = *reinterpret_cast<const Quad<T>*>(p + (ok ? row0 + i : 0));
#pragma unroll
            for (int e = 0; e < 4; e++) dst[i + e] = ok ? ld_f32(&t.v[e]) : 0.f;
        }
    } else {
#pragma unroll
        for (int i = 0; i < R; i++) {
            const float x = ld_f32(p + min(row0 + i, rows - 1));
            dst[i] = row0 + i < rows ? x : 0.f;
        }
    }
}
}  // namespace

// ---- token by token.  grid (sequences, heads, blocks of 16 columns), one wave ---------------------------------------------
// R: rows a lane keeps (16 R >= dk)
template <typename T, int R, bool VEC>
__global__ void __launch_bounds__(64)
delta_rows_k(DeltaArgs x) {
    const int seq = blockIdx.x, h = blockIdx.y, lane = threadIdx.x, row0 = (lane >> 2) * R, c0 = blockIdx.z * 16 + (lane & 3) * 4;
    const int H = x.H, dk = x.dk, dv = x.dv, kvh = h / (H / x.G);
    const int begin = x.cu_rows[seq], end = x.cu_rows[seq + 1];
    if (begin >= end) return;
    float* st = x.state + ((size_t)x.slot_ids[seq] * H + h) * dk * dv;
    const T* qp = (const T*)x.q + (size_t)kvh * dk;
    const T* kp = (const T*)x.k + (size_t)kvh * dk;
    const T* vp = (const T*)x.v + (size_t)h * dv;
    const bool quads = dv % 4 == 0;
    float S[R][4];
#pragma unroll
    for (int i = 0; i < R; i++) {
        const int row = row0 + i, rc = min(row, dk - 1);
        if (quads) {
            const float4 t = *reinterpret_cast<const float4*>(st + (size_t)rc * dv + min(c0, dv - 4));
            S[i][0] = t.x; S[i][1] = t.y; S[i][2] = t.z; S[i][3] = t.w;
        } else {
#pragma unroll
            for (int e = 0; e < 4; e++) S[i][e] = st[(size_t)rc * dv + min(c0 + e, dv - 1)];
        }
#pragma unroll
        for (int e = 0; e < 4; e++) if (row >= dk || c0 + e >= dv) S[i][e] = 0.f;
    }
    const float a_log = x.a_log[h], dt_bias = x.dt_bias[h];
    float qn[R], kn[R], vn[4], an, bn;
    auto fetch = [&](int t) {
        t = min(t, end - 1);                             // past the end: a row that exists, never used
        load_part<T, R, VEC>(qn, qp + (size_t)t * x.q_stride, row0, dk);
        load_part<T, R, VEC>(kn, kp + (size_t)t * x.k_stride, row0, dk);
#pragma unroll
        for (int e = 0; e < 4; e++) vn[e] = ld_f32(vp + (size_t)t * x.v_stride + min(c0 + e, dv - 1));
        an = ld_f32((const T*)x.a + (size_t)t * x.gate_stride + h);
        bn = ld_f32((const T*)x.b + (size_t)t * x.gate_stride + h);
    };
    fetch(begin);
    for (int t = begin; t < end; t++) {
        float q[R], k[R], v[4];
#pragma unroll
        for (int i = 0; i < R; i++) { q[i] = qn[i]; k[i] = kn[i]; }
#pragma unroll
        for (int e = 0; e < 4; e++) v[e] = vn[e];
        const float g = expf(log_decay_of(an, dt_bias, a_log)), beta = step_of(bn);
        fetch(t + 1);
        float kk = 0.f, qq = 0.f, qk = 0.f, dk_[4] = {}, dq_[4] = {};
#pragma unroll
        for (int i = 0; i < R; i++) {
            kk = __builtin_fmaf(k[i], k[i], kk);
            qq = __builtin_fmaf(q[i], q[i], qq);
            qk = __builtin_fmaf(q[i], k[i], qk);
#pragma unroll
            for (int e = 0; e < 4; e++) {
                dk_[e] = __builtin_fmaf(k[i], S[i][e], dk_[e]);
                dq_[e] = __builtin_fmaf(q[i], S[i][e], dq_[e]);
            }
        }
        const float ik = rsqrtf(rows_sum(kk) + UNIT_EPS), iq = rsqrtf(rows_sum(qq) + UNIT_EPS) * x.q_scale;
        qk = rows_sum(qk) * ik * iq;
        float o[4], ku[4];
#pragma unroll
        for (int e = 0; e < 4; e++) {
            const float u = beta * (v[e] - g * ik * rows_sum(dk_[e]));
            o[e] = __builtin_fmaf(qk, u, g * iq * rows_sum(dq_[e]));         // S^T q after the write: g S_old^T q + (q . k) u
            ku[e] = ik * u;
        }
#pragma unroll
        for (int i = 0; i < R; i++)
#pragma unroll
            for (int e = 0; e < 4; e++) S[i][e] = __builtin_fmaf(k[i], ku[e], g * S[i][e]);
        if (lane < 4) {
            float* yr = x.y + ((size_t)t * H + h) * dv + c0;
#pragma unroll
            for (int e = 0; e < 4; e++) if (c0 + e < dv) yr[e] = o[e];
        }
    }
#pragma unroll
    for (int i = 0; i < R; i++) {
        const int row = row0 + i;
        if (row >= dk) continue;
        if (quads) { if (c0 < dv) *reinterpret_cast<float4*>(st + (size_t)row * dv + c0) = make_float4(S[i][0], S[i][1], S[i][2], S[i][3]); }
        else {
#pragma unroll
            for (int e = 0; e < 4; e++) if (c0 + e < dv) st[(size_t)row * dv + c0 + e] = S[i][e];
        }
    }
}

// ---- chunks --------------------------------------------------------------------------------------------------------------
namespace {
union DFrag { uint4 u; dl_bf16x8 v; bf16_t h[8]; };
typedef __attribute__((__vector_size__(2 * sizeof(float)))) float dl_f32x2;
typedef __attribute__((__vector_size__(2 * sizeof(__bf16)))) __bf16 dl_bf16x2;
// a and b as sums of three bfloat16 numbers, to float32's 24 bits: word n holds their nth terms
__device__ __forceinline__ void split_pair(float a, float b, uint32_t (&word)[3]) {
#pragma unroll
    for (int n = 0; n < 3; n++) {
        word[n] = __builtin_bit_cast(uint32_t, __builtin_convertvector((dl_f32x2){a, b}, dl_bf16x2));
        a -= __uint_as_float(word[n] << 16);
        b -= __uint_as_float(word[n] & 0xffff0000u);
    }
}
// four neighbouring elements of a row of terms, term n at dst + n * apart
__device__ __forceinline__ void put4(bf16_t* dst, int apart, float f0, float f1, float f2, float f3) {
    uint32_t lo[3], hi[3];
    split_pair(f0, f1, lo);
    split_pair(f2, f3, hi);
#pragma unroll
    for (int n = 0; n < 3; n++) *reinterpret_cast<uint2*>(dst + n * apart) = make_uint2(lo[n], hi[n]);
}
__device__ __forceinline__ dl_f32x4 mma(const DFrag& a, const DFrag& b, dl_f32x4 c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.v, b.v, c, 0, 0, 0);
}
// (a0 + a1 + a2)(b0 + b1 + b2) without the products below 2^-24 of the whole, in two chains of sums
__device__ __forceinline__ void mma_terms(const DFrag (&a)[3], const DFrag (&b)[3], dl_f32x4& c, dl_f32x4& d) {
    c = mma(a[0], b[2], c); d = mma(a[1], b[1], d);
    c = mma(a[2], b[0], c); d = mma(a[0], b[1], d);
    c = mma(a[1], b[0], c); d = mma(a[0], b[0], d);
}
// A barrier for what the waves pass through LDS.  (__syncthreads() would also wait for every load from memory that is
// under way, and a chunk's loads are asked for a chunk ahead.)
__device__ __forceinline__ void lds_barrier() { asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory"); }
// where head h of (sequence, chunk) c keeps its two matrices' terms, its scalars, and the kv head's K transposed
__device__ __forceinline__ bf16_t* ws_terms(const DeltaArgs& x, size_t c, int h, int which) { return x.ws_mat + ((c * x.H + h) * 2 + which) * 3 * DC * DC; }
__device__ __forceinline__ float* ws_scalars(const DeltaArgs& x, size_t c, int h) { return x.ws_scal + (c * x.H + h) * 4 * DC; }
}  // namespace

// grid (sequences x chunks, heads), four waves: wave w forms the rows 16 w .. 16 w + 15 of the two 64 x 64 matrices
template <int KS>
__global__ void __launch_bounds__(256)
delta_prepare_k(DeltaArgs x) {
    constexpr int LS = DC + 4, KP = KS * 32 + 8;
    __shared__ __attribute__((aligned(16))) float Ls[DC * LS];        // L, then the inverse of I + L
    __shared__ __attribute__((aligned(16))) float As[DC * LS];        // A
    __shared__ __attribute__((aligned(16))) bf16_t Kr[DC * KP], Kt[KS * 32 * DCP];      // the chunk's keys by rows, and transposed
    __shared__ double Gs[DC];
    __shared__ float beta_s[DC], ik_s[DC], iq_s[DC];
    const int seq = blockIdx.x / x.n_chunks, chunk = blockIdx.x % x.n_chunks, h = blockIdx.y;
    const int begin = x.cu_rows[seq] + chunk * DC, n = min(DC, x.cu_rows[seq + 1] - begin);
    if (n <= 0) return;
    const int per = x.H / x.G, kvh = h / per, dk = x.dk;
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, r = lane & 15, g = lane >> 4;
    // the wave's 16 rows of K and Q (a row past the chunk's end: its last row once more, of a token whose step is zero)
    const size_t at = (size_t)(begin + min(wave * 16 + r, n - 1));
    const bf16_t* kp = (const bf16_t*)x.k + at * x.k_stride + (size_t)kvh * dk;
    const bf16_t* qp = (const bf16_t*)x.q + at * x.q_stride + (size_t)kvh * dk;
    DFrag kf[KS], qf[KS];
#pragma unroll
    for (int s = 0; s < KS; s++) {
        const int d = min(s * 32 + g * 8, dk - 8);
        kf[s].u = *reinterpret_cast<const uint4*>(kp + d);
        qf[s].u = *reinterpret_cast<const uint4*>(qp + d);
    }
    if (wave == 0) {                                     // the tokens' decays and steps, a token a lane
        double G = 0.0;
        float beta = 0.f;
        if (lane < n) {
            const size_t at = (size_t)(begin + lane) * x.gate_stride + h;
            G = (double)log_decay_of(bf16_to_f32(((const bf16_t*)x.a)[at]), x.dt_bias[h], x.a_log[h]);
            beta = step_of(bf16_to_f32(((const bf16_t*)x.b)[at]));
        }
#pragma unroll
        for (int o = 1; o < 64; o <<= 1) {
            const double up = __shfl_up(G, o, 64);
            if (lane >= o) G += up;
        }
        Gs[lane] = G;
        beta_s[lane] = beta;
    }
    if (dk < KS * 32) {                                  // elements past the head's are zeros
        const uint4 zero = make_uint4(0, 0, 0, 0);
#pragma unroll
        for (int s = 0; s < KS; s++)
            if (s * 32 + g * 8 >= dk) { kf[s].u = zero; qf[s].u = zero; }
    }
#pragma unroll
    for (int s = 0; s < KS; s++) *reinterpret_cast<uint4*>(Kr + (wave * 16 + r) * KP + s * 32 + g * 8) = kf[s].u;
    {
        float kk = 0.f, qq = 0.f;
#pragma unroll
        for (int s = 0; s < KS; s++)
#pragma unroll
            for (int e = 0; e < 8; e++) {
                const float a = bf16_to_f32(kf[s].h[e]), b = bf16_to_f32(qf[s].h[e]);
                kk = __builtin_fmaf(a, a, kk);
                qq = __builtin_fmaf(b, b, qq);
            }
        kk += __shfl_xor(kk, 16, 64); kk += __shfl_xor(kk, 32, 64);
        qq += __shfl_xor(qq, 16, 64); qq += __shfl_xor(qq, 32, 64);
        if (g == 0) {
            ik_s[wave * 16 + r] = rsqrtf(kk + UNIT_EPS);
            iq_s[wave * 16 + r] = rsqrtf(qq + UNIT_EPS) * x.q_scale;
        }
    }
    const bool transposes = h % per == 0;                // one head of a group turns the shared keys
    if (transposes)
#pragma unroll
        for (int s = 0; s < KS; s++)
#pragma unroll
            for (int e = 0; e < 8; e++) Kt[(s * 32 + g * 8 + e) * DCP + wave * 16 + r] = kf[s].h[e];
    __syncthreads();
    for (int j = 0; j < 4; j++) {                        // tile (wave, j): tokens t = 16 wave + 4 g + i against s = 16 j + r
        dl_f32x4 kkt = {0.f, 0.f, 0.f, 0.f}, qkt = {0.f, 0.f, 0.f, 0.f};
        if (j <= wave) {
#pragma unroll
            for (int s = 0; s < KS; s++) {
                DFrag kb;
                kb.u = *reinterpret_cast<const uint4*>(Kr + (j * 16 + r) * KP + s * 32 + g * 8);
                kkt = mma(kf[s], kb, kkt);
                qkt = mma(qf[s], kb, qkt);
            }
        }
        const int ss = j * 16 + r;
        const double Gss = Gs[ss];
        const float iks = ik_s[ss];
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const int t = wave * 16 + g * 4 + i;
            const float decay = ss <= t ? expf((float)(Gs[t] - Gss)) : 0.f;
            Ls[t * LS + ss] = ss < t ? beta_s[t] * decay * ik_s[t] * iks * kkt[i] : 0.f;
            As[t * LS + ss] = ss <= t ? decay * iq_s[t] * iks * qkt[i] : 0.f;
        }
    }
    __syncthreads();
    // The inverse of I + L by blocks of 16: wave w inverts the diagonal block w, a column a lane, then the blocks left of it,
    // one diagonal after the other:  T_wj = -T_ww (sum over k = j .. w - 1 of L_wk T_kj).  A wave holds its rows of L, so
    // that T may take L's place.  The products are float32 ones; a result's rows 4 g + i are the k of its next use at step i.
    dl_f32x4 Lf[3];                                      // L_wk, lane: row r, columns 4 g + i
#pragma unroll
    for (int k = 0; k < 3; k++)
        if (k < wave) {
            const float4 l = *reinterpret_cast<const float4*>(Ls + (wave * 16 + r) * LS + k * 16 + g * 4);
            Lf[k] = (dl_f32x4){l.x, l.y, l.z, l.w};
        }
    {
        float T[16];
#pragma unroll
        for (int t = 0; t < 16; t++) {
            float s0 = 0.f, s1 = 0.f;
#pragma unroll
            for (int c = 0; c < t; c += 4) {
                const float4 l = *reinterpret_cast<const float4*>(Ls + (wave * 16 + t) * LS + wave * 16 + c);     // zero from c = t on
                s0 = __builtin_fmaf(l.x, T[c], s0);
                if (c + 1 < t) s1 = __builtin_fmaf(l.y, T[c + 1], s1);
                if (c + 2 < t) s0 = __builtin_fmaf(l.z, T[c + 2], s0);
                if (c + 3 < t) s1 = __builtin_fmaf(l.w, T[c + 3], s1);
            }
            T[t] = (t == r ? 1.f : 0.f) - (s0 + s1);
        }
        if (g == 0)
#pragma unroll
            for (int t = 0; t < 16; t++) Ls[(wave * 16 + t) * LS + wave * 16 + r] = T[t];
    }
    if (wave == 1) {
        float* sc = ws_scalars(x, blockIdx.x, h);
        const double G = Gs[lane], end = Gs[DC - 1];
        const float eg = expf((float)G);
        sc[lane] = eg * ik_s[lane];
        sc[DC + lane] = eg * iq_s[lane];
        sc[2 * DC + lane] = expf((float)(end - G)) * ik_s[lane];
        sc[3 * DC + lane] = expf((float)end);
    }
    if (transposes) {
        bf16_t* kt = x.ws_kt + ((size_t)blockIdx.x * x.G + kvh) * x.dkp * DC;
        for (int i = tid; i < KS * 32 * 8; i += 256) {
            const int d = i >> 3, c = (i & 7) * 8;
            *reinterpret_cast<uint4*>(kt + d * DC + c) = *reinterpret_cast<const uint4*>(Kt + d * DCP + c);
        }
    }
    __syncthreads();
#pragma unroll
    for (int d = 1; d < 4; d++) {
        const int j = wave - d;
        if (j >= 0) {
            dl_f32x4 sum = {0.f, 0.f, 0.f, 0.f}, t = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int k = 0; k < 3; k++)
                if (k >= j && k < wave)
#pragma unroll
                    for (int i = 0; i < 4; i++)
                        sum = __builtin_amdgcn_mfma_f32_16x16x4f32(Lf[k][i], Ls[(k * 16 + g * 4 + i) * LS + j * 16 + r], sum, 0, 0, 0);
#pragma unroll
            for (int i = 0; i < 4; i++)
                t = __builtin_amdgcn_mfma_f32_16x16x4f32(-Ls[(wave * 16 + r) * LS + wave * 16 + g * 4 + i], sum[i], t, 0, 0, 0);
#pragma unroll
            for (int i = 0; i < 4; i++) Ls[(wave * 16 + g * 4 + i) * LS + j * 16 + r] = t[i];
        }
        __syncthreads();
    }
    // the two matrices in terms: a thread takes 16 columns of a row
    const int row = tid >> 2, col = (tid & 3) * 16;
    if (col < 32 * (row / 32 + 1)) {                     // what a row of tiles is multiplied by: whole k steps up to its diagonal
#pragma unroll
        for (int which = 0; which < 2; which++) {
            const float* src = (which ? As : Ls) + row * LS + col;
            bf16_t* dst = ws_terms(x, blockIdx.x, h, which) + row * DC + col;
#pragma unroll
            for (int e = 0; e < 16; e += 4) {
                float4 f = *reinterpret_cast<const float4*>(src + e);
                if (which == 0) { f.x *= beta_s[col + e]; f.y *= beta_s[col + e + 1]; f.z *= beta_s[col + e + 2]; f.w *= beta_s[col + e + 3]; }
                put4(dst + e, DC * DC, f.x, f.y, f.z, f.w);
            }
        }
    }
}

// grid (8 dies x units of a (sequence, head) a die takes x blocks of 16 columns), four waves: wave w takes the tokens 16 w .. 16 w + 15 of a chunk and the 16-row
// tiles w, w + 4, .. of the state, which it keeps in float32; the state's terms, R = V - diag(e^G) K S_0 and U pass between the
// waves through LDS.
template <int KS>
__global__ void __launch_bounds__(256)
delta_chunks_k(DeltaArgs x) {
    constexpr int DKP = KS * 32, SP = DKP + 8, TILES = (2 * KS + 3) / 4;
    __shared__ __attribute__((aligned(16))) bf16_t S_lds[3][16][SP];
    __shared__ __attribute__((aligned(16))) bf16_t R_lds[3][16][DCP], U_lds[3][16][DCP], C_lds[3][16][DCP];
    // blocks of one head follow one another on one of the eight dies (block b runs on die b % 8), so that a chunk's matrices
    // and keys come from its cache for all but the first
    const int places = (x.n_seq * x.H + 7) / 8, blocks_h = (x.dv + 15) / 16, slot = blockIdx.x >> 3;
    const int unit = (blockIdx.x & 7) * places + slot / blocks_h;
    if (unit >= x.n_seq * x.H) return;
    const int seq = unit / x.H, h = unit % x.H, c0 = slot % blocks_h * 16;
    const int row_first = x.cu_rows[seq], count = x.cu_rows[seq + 1] - row_first;
    if (count <= 0) return;
    const int kvh = h / (x.H / x.G), dk = x.dk, dv = x.dv;
    const int tid = threadIdx.x, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lane = tid & 63, r = lane & 15, g = lane >> 4;
    const int col = c0 + r, colc = min(col, dv - 1);
    float* st = x.state + ((size_t)x.slot_ids[seq] * x.H + h) * dk * dv;
    dl_f32x4 S[TILES];
#pragma unroll
    for (int j = 0; j < TILES; j++) {
        const int tile = wave + 4 * j;
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const int row = tile * 16 + g * 4 + i;
            const float s = st[(size_t)min(row, dk - 1) * dv + colc];
            S[j][i] = row < dk && col < dv ? s : 0.f;
        }
        if (tile < 2 * KS) put4(&S_lds[0][r][tile * 16 + g * 4], 16 * SP, S[j][0], S[j][1], S[j][2], S[j][3]);
    }
    // What a chunk needs from memory is asked for a chunk ahead, into the registers it has just left, by loads without a
    // condition: rows past the sequence's end and elements past a head's read something that exists.  It comes to nothing: such
    // a token's step is zero (its U with it), the state's rows past dk are zero, and neither is stored.
    const int n_chunks = (count + DC - 1) / DC;
    const size_t c_first = (size_t)seq * x.n_chunks;
    DFrag kf[KS], qf[KS], tf[2][3], af[2][3], ktf[TILES][2];
    bf16_t v[4];
    float4 ka, qa, kc, ka_next, qa_next, kc_next;
    float all, all_next;
    const char* const q_seq = (const char*)((const bf16_t*)x.q + (size_t)row_first * x.q_stride + (size_t)kvh * dk);
    const char* const k_seq = (const char*)((const bf16_t*)x.k + (size_t)row_first * x.k_stride + (size_t)kvh * dk);
    const char* const v_seq = (const char*)((const bf16_t*)x.v + (size_t)row_first * x.v_stride + (size_t)h * dv);
    auto rows_of = [&](int c) {                          // K, Q and V of the wave's 16 tokens
        const int first = c * DC, last = count - 1 - first;
        const char* kb = k_seq + (size_t)first * x.k_stride * 2;
        const char* qb = q_seq + (size_t)first * x.q_stride * 2;
        const char* vb = v_seq + (size_t)first * x.v_stride * 2;
        const unsigned t = (unsigned)min(wave * 16 + r, last);
        const unsigned ko = t * (unsigned)x.k_stride * 2u, qo = t * (unsigned)x.q_stride * 2u;
#pragma unroll
        for (int s = 0; s < KS; s++) {
            const unsigned d = (unsigned)min(s * 32 + g * 8, dk - 8) * 2u;
            kf[s].u = *reinterpret_cast<const uint4*>(kb + (ko + d));
            qf[s].u = *reinterpret_cast<const uint4*>(qb + (qo + d));
        }
#pragma unroll
        for (int i = 0; i < 4; i++)
            v[i] = *reinterpret_cast<const bf16_t*>(vb + ((unsigned)min(wave * 16 + g * 4 + i, last) * (unsigned)x.v_stride + (unsigned)colc) * 2u);
    };
    auto scalars_of = [&](size_t c) {
        const float* sc = ws_scalars(x, c, h) + wave * 16;
        ka_next = *reinterpret_cast<const float4*>(sc + g * 4);
        qa_next = *reinterpret_cast<const float4*>(sc + DC + g * 4);
        kc_next = *reinterpret_cast<const float4*>(sc + 2 * DC + g * 4);
        all_next = sc[3 * DC + r];
    };
    const unsigned term_at = (unsigned)((wave * 16 + r) * DC + g * 8) * 2u;
    auto terms_of = [&](size_t c, int which, DFrag (&f)[2][3]) {
        const char* p = (const char*)ws_terms(x, c, h, which);
#pragma unroll
        for (int s = 0; s < 2; s++)
#pragma unroll
            for (int n = 0; n < 3; n++) f[s][n].u = *reinterpret_cast<const uint4*>(p + (term_at + (unsigned)(n * DC * DC + s * 32) * 2u));
    };
    auto keys_of = [&](size_t c) {
        const char* p = (const char*)(x.ws_kt + (c * x.G + kvh) * x.dkp * DC);
#pragma unroll
        for (int j = 0; j < TILES; j++)
#pragma unroll
            for (int s = 0; s < 2; s++)
                ktf[j][s].u = *reinterpret_cast<const uint4*>(p + (unsigned)((min(wave + 4 * j, 2 * KS - 1) * 16 + r) * DC + g * 8 + s * 32) * 2u);
    };
    rows_of(0);
    scalars_of(c_first);
    terms_of(c_first, 0, tf);
    keys_of(c_first);
    terms_of(c_first, 1, af);
    lds_barrier();
    const bool both = wave >= 2;                         // the upper two waves' rows of the matrices reach into the second k step
    for (int c = 0; c < n_chunks; c++) {
        const int next = min(c + 1, n_chunks - 1);       // (after the last chunk: once more what is there)
        ka = ka_next; qa = qa_next; kc = kc_next; all = all_next;
        // K S_0 and Q S_0
        dl_f32x4 ks[2], qs[2];
#pragma unroll
        for (int i = 0; i < 2; i++) { ks[i] = (dl_f32x4){0.f, 0.f, 0.f, 0.f}; qs[i] = ks[i]; }
#pragma unroll
        for (int n = 2; n >= 0; n--)
#pragma unroll
            for (int s = 0; s < KS; s++) {
                DFrag b;
                b.u = *reinterpret_cast<const uint4*>(&S_lds[n][r][s * 32 + g * 8]);
                ks[s & 1] = mma(kf[s], b, ks[s & 1]);
                qs[s & 1] = mma(qf[s], b, qs[s & 1]);
            }
        ks[0] = ks[0] + ks[1];
        put4(&R_lds[0][r][wave * 16 + g * 4], 16 * DCP, bf16_to_f32(v[0]) - ka.x * ks[0][0], bf16_to_f32(v[1]) - ka.y * ks[0][1],
             bf16_to_f32(v[2]) - ka.z * ks[0][2], bf16_to_f32(v[3]) - ka.w * ks[0][3]);
        qs[0] = qs[0] + qs[1];
        dl_f32x4 o = {qa.x * qs[0][0], qa.y * qs[0][1], qa.z * qs[0][2], qa.w * qs[0][3]}, o1 = {0.f, 0.f, 0.f, 0.f};
        rows_of(next);
        scalars_of(c_first + next);
        lds_barrier();
        dl_f32x4 u = {0.f, 0.f, 0.f, 0.f}, u1 = u;
#pragma unroll
        for (int s = 0; s < 2; s++)
            if (s == 0 || both) {
                DFrag b[3];
#pragma unroll
                for (int n = 0; n < 3; n++) b[n].u = *reinterpret_cast<const uint4*>(&R_lds[n][r][s * 32 + g * 8]);
                mma_terms(tf[s], b, u, u1);
            }
        u = u + u1;
        terms_of(c_first + next, 0, tf);
        put4(&C_lds[0][r][wave * 16 + g * 4], 16 * DCP, kc.x * u[0], kc.y * u[1], kc.z * u[2], kc.w * u[3]);
        put4(&U_lds[0][r][wave * 16 + g * 4], 16 * DCP, u[0], u[1], u[2], u[3]);
#pragma unroll
        for (int j = 0; j < TILES; j++) S[j] = S[j] * all;
        lds_barrier();
#pragma unroll
        for (int s = 0; s < 2; s++) {
            DFrag b[3];
#pragma unroll
            for (int n = 0; n < 3; n++) b[n].u = *reinterpret_cast<const uint4*>(&C_lds[n][r][s * 32 + g * 8]);
#pragma unroll
            for (int n = 2; n >= 0; n--)
#pragma unroll
                for (int j = 0; j < TILES; j++) S[j] = mma(ktf[j][s], b[n], S[j]);
        }
        keys_of(c_first + next);
#pragma unroll
        for (int j = 0; j < TILES; j++)
            if (2 * KS % 4 == 0 || wave + 4 * j < 2 * KS) put4(&S_lds[0][r][(wave + 4 * j) * 16 + g * 4], 16 * SP, S[j][0], S[j][1], S[j][2], S[j][3]);
#pragma unroll
        for (int s = 0; s < 2; s++)
            if (s == 0 || both) {
                DFrag b[3];
#pragma unroll
                for (int n = 0; n < 3; n++) b[n].u = *reinterpret_cast<const uint4*>(&U_lds[n][r][s * 32 + g * 8]);
                mma_terms(af[s], b, o, o1);
            }
        terms_of(c_first + next, 1, af);
        o = o + o1;
        const int t0 = c * DC + wave * 16 + g * 4;
        float* yr = x.y + ((size_t)(row_first + t0) * x.H + h) * dv + col;
#pragma unroll
        for (int i = 0; i < 4; i++) if (t0 + i < count && col < dv) yr[(size_t)i * x.H * dv] = o[i];
        lds_barrier();
    }
#pragma unroll
    for (int j = 0; j < TILES; j++)
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const int row = (wave + 4 * j) * 16 + g * 4 + i;
            if (row < dk && col < dv) st[(size_t)row * dv + col] = S[j][i];
        }
}

static int delta_dkp(int dk) { const int s = tp_cdiv(dk, 32); return 32 * (s <= 4 ? s : (s <= 6 ? 6 : 8)); }     // key rows the chunks' kernels are made for
static size_t delta_align(size_t n) { return (n + 255) / 256 * 256; }
static size_t delta_mat_bytes(long units) { return delta_align((size_t)units * 2 * 3 * DC * DC * sizeof(bf16_t)); }
static size_t delta_scal_bytes(long units) { return delta_align((size_t)units * 4 * DC * sizeof(float)); }

// bytes of workspace for steps that run in chunks (n_chunks of 64 tokens cover the longest sequence)
extern "C" long tp_delta_scan_workspace_bytes(int n_seq, int n_chunks, int H, int G, int dk) {
    const long units = (long)n_seq * n_chunks * H;
    return (long)(delta_mat_bytes(units) + delta_scal_bytes(units) + delta_align((size_t)n_seq * n_chunks * G * delta_dkp(dk) * DC * sizeof(bf16_t)));
}

// q, k [M, G dk], v [M, H dv], b, a [M, H] as views of wider rows, all of one dtype; state [slots, H, dk, dv] float32, left
// updated; y float32 [M, H dv].  n_chunks > 0: bfloat16 steps in chunks of 64 tokens, that many covering the longest sequence.
extern "C" int tp_delta_scan(const void* q, long q_stride, const void* k, long k_stride, const void* v, long v_stride, const void* b,
                             const void* a, long gate_stride, int dtype, const float* a_log, const float* dt_bias, float* state,
                             const int* slot_ids, const int* cu_rows, float* y, int n_seq, int H, int G, int dk, int dv, float q_scale,
                             int n_chunks, void* workspace, long workspace_bytes, void* stream) {
    TP_REQUIRE(n_seq > 0 && H > 0 && G > 0 && dk > 0 && dv > 0, "delta_scan: empty shape sequences=%d heads=%d kv=%d key=%d value=%d", n_seq, H, G, dk, dv);
    TP_REQUIRE(H % G == 0, "delta_scan: %d heads are no multiple of %d kv heads", H, G);
    TP_REQUIRE(dk <= 256, "delta_scan: keys of %d elements exceed 256", dk);
    TP_REQUIRE(H <= 65535 && tp_cdiv(dv, 16) <= 65535, "delta_scan: %d heads of %d values exceed one launch", H, dv);
    TP_REQUIRE(q && k && v && b && a && a_log && dt_bias && state && slot_ids && cu_rows && y, "delta_scan: null operand");
    TP_REQUIRE(dtype == TP_BF16 || dtype == TP_F32, "delta_scan: unknown dtype %d", dtype);
    hipStream_t s = (hipStream_t)stream;
    DeltaArgs x{q, q_stride, k, k_stride, v, v_stride, b, a, gate_stride, a_log, dt_bias, state, slot_ids, cu_rows, y, n_seq, H, G, dk, dv, q_scale,
                0, 0, nullptr, nullptr, nullptr};
    dim3 grid(n_seq, H, tp_cdiv(dv, 16));
    if (n_chunks > 0) {
        TP_REQUIRE(dtype == TP_BF16 && dk % 8 == 0 && q_stride % 8 == 0 && k_stride % 8 == 0 && (uintptr_t)q % 16 == 0 && (uintptr_t)k % 16 == 0,
                   "delta_scan: chunks need bfloat16 rows of whole 16-byte pieces");
        TP_REQUIRE((long)n_seq * n_chunks <= 0x7fffffffL, "delta_scan: %d chunks of %d sequences exceed one launch", n_chunks, n_seq);
        TP_REQUIRE(workspace && (uintptr_t)workspace % 16 == 0 && workspace_bytes >= tp_delta_scan_workspace_bytes(n_seq, n_chunks, H, G, dk), "delta_scan: a workspace of %ld bytes is too small", workspace_bytes);
        const long units = (long)n_seq * n_chunks * H;
        x.n_chunks = n_chunks;
        x.dkp = delta_dkp(dk);
        x.ws_mat = (bf16_t*)workspace;
        x.ws_scal = (float*)((char*)workspace + delta_mat_bytes(units));
        x.ws_kt = (bf16_t*)((char*)x.ws_scal + delta_scal_bytes(units));
        dim3 pgrid(n_seq * n_chunks, H);
        const long cgrid = 8L * ((n_seq * (long)H + 7) / 8) * tp_cdiv(dv, 16);
        TP_REQUIRE(cgrid <= 0x7fffffffL, "delta_scan: %ld blocks exceed one launch", cgrid);
#define TP_DELTA_CHUNKS(KS) do { delta_prepare_k<KS><<<pgrid, 256, 0, s>>>(x); delta_chunks_k<KS><<<(unsigned)cgrid, 256, 0, s>>>(x); } while (0)
        switch (x.dkp / 32) {
            case 1: TP_DELTA_CHUNKS(1); break;
            case 2: TP_DELTA_CHUNKS(2); break;
            case 3: TP_DELTA_CHUNKS(3); break;
            case 4: TP_DELTA_CHUNKS(4); break;
            case 6: TP_DELTA_CHUNKS(6); break;
            default: TP_DELTA_CHUNKS(8); break;
        }
#undef TP_DELTA_CHUNKS
        return tp_check_launch("delta_scan (chunks)");
    }
    const long el = dtype == TP_BF16 ? 2 : 4;
    const bool vec = dk % 4 == 0 && q_stride % 4 == 0 && k_stride % 4 == 0 && (uintptr_t)q % (4 * el) == 0 && (uintptr_t)k % (4 * el) == 0;
#define TP_DELTA_ROWS(R) do { \
        if (dtype == TP_BF16) { if (vec) delta_rows_k<bf16_t, R, true><<<grid, 64, 0, s>>>(x); else delta_rows_k<bf16_t, R, false><<<grid, 64, 0, s>>>(x); } \
        else { if (vec) delta_rows_k<float, R, true><<<grid, 64, 0, s>>>(x); else delta_rows_k<float, R, false><<<grid, 64, 0, s>>>(x); } } while (0)
    if (dk <= 64) TP_DELTA_ROWS(4);
    else if (dk <= 128) TP_DELTA_ROWS(8);
    else TP_DELTA_ROWS(16);
#undef TP_DELTA_ROWS
    return tp_check_launch("delta_scan");
}
