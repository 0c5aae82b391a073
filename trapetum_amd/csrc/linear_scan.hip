// Linear attention whose memory decays by a constant per head.
//
//   per head, token by token:   S <- g S + v k^T,   o = S q        (S is dv x dk, zero before the sequence, g a constant)
//
// S, the powers of g and every sum are float32; q, k and v arrive as the projection left them (bfloat16 in a bfloat16
// engine).  A row of S (one value element) goes on by itself.
//
// Two forms.  `scan_rows_k` takes a sequence's tokens one by one: 16 rows of S a wave, 4 lanes a row (a decode step, short
// portions, float32 engines).  Long bfloat16 steps run in chunks of 64 tokens on the matrix cores.  The decay is the same
// for every token, so the chunks do not wait for one another: with n tokens in a chunk and S_0 the state it starts from,
//   E   = sum_t g^(n - 1 - t) v_t k_t^T                       scan_ends_k: what the chunk leaves behind, all chunks at once
//   S_0 of the next chunk = g^n S_0 + E                       scan_carry_k: element by element along the chunks
//   o_t = g^(t + 1) S_0 q_t + sum_(s <= t) g^(t - s) (k_s . q_t) v_s        scan_outputs_k: all chunks at once
// A float32 operand of a matrix product (E's decayed values, S_0, the weights g^(t - s) (k_s . q_t)) is split into three
// bfloat16 terms, which keep its 24 bits; the other operand is bfloat16 as it is; sums are float32.
#include "common.h"

typedef __attribute__((__vector_size__(8 * sizeof(__bf16)))) __bf16 ls_bf16x8;
typedef __attribute__((__vector_size__(4 * sizeof(float)))) float ls_f32x4;
typedef __attribute__((__vector_size__(2 * sizeof(float)))) float ls_f32x2;
typedef __attribute__((__vector_size__(2 * sizeof(__bf16)))) __bf16 ls_bf16x2;

struct LinearScanArgs {
    const void* q; long q_stride; const void* k; long k_stride; const void* v; long v_stride;
    const float* decay;                                  // [H]
    float* state;                                        // [slots, H, dv, dk]
    const int* slot_ids; const int* cu_rows; float* y;   // y [M, H dv]
    int n_seq, H, dk, dv;
    int n_chunks;                                        // chunks of the longest sequence
    float* chunks;                                       // [sequence x chunk, H, dv, dk]: E, which gives way to S_0
};

namespace {
constexpr int LC = 64;                           // tokens of a chunk
constexpr int LCP = LC + 8;                      // a row of 64 tokens in LDS
constexpr int EB = 64;                           // value elements a block of scan_ends_k takes
template <typename T> struct alignas(sizeof(T) * 4) Four { T v[4]; };
union LFrag { uint4 u; ls_bf16x8 v; uint32_t w[4]; };

// a and b as sums of three bfloat16 numbers: word n holds their nth terms
__device__ __forceinline__ void split_two(float a, float b, uint32_t (&word)[3]) {
#pragma unroll
    for (int n = 0; n < 3; n++) {
        word[n] = __builtin_bit_cast(uint32_t, __builtin_convertvector((ls_f32x2){a, b}, ls_bf16x2));
        a -= __uint_as_float(word[n] << 16);
        b -= __uint_as_float(word[n] & 0xffff0000u);
    }
}
__device__ __forceinline__ ls_f32x4 mma(const LFrag& a, const LFrag& b, ls_f32x4 c) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.v, b.v, c, 0, 0, 0);
}
__device__ __forceinline__ float power(float g, int n) { return n == 0 ? 1.f : powf(g, (float)n); }
}  // namespace

// ---- token by token.  grid (sequences, heads, blocks of 16 value elements), one wave: lane l holds row l / 4 of the block's
// 16, and of it the quads 4 j + l % 4 (NJ of them: 16 NJ >= dk) --------------------------------------------------------------
template <typename T, int NJ, bool VEC>
__global__ void __launch_bounds__(64)
scan_rows_k(LinearScanArgs x) {
    const int seq = blockIdx.x, h = blockIdx.y, lane = threadIdx.x, e = blockIdx.z * 16 + (lane >> 2), d0 = (lane & 3) * 4;
    const int H = x.H, dk = x.dk, dv = x.dv, ec = min(e, dv - 1);
    const int begin = x.cu_rows[seq], end = x.cu_rows[seq + 1];
    if (begin >= end) return;
    float* st = x.state + (((size_t)x.slot_ids[seq] * H + h) * dv + ec) * dk;
    const T* qp = (const T*)x.q + (size_t)h * dk;
    const T* kp = (const T*)x.k + (size_t)h * dk;
    const T* vp = (const T*)x.v + (size_t)h * dv + ec;
    const float g = x.decay[h];
    float S[NJ][4], kn[NJ][4], qn[NJ][4], vn;
    auto row4 = [&](const T* p, float (&o)[NJ][4]) {       // a lane's elements of a row, zeros past its end
#pragma unroll
        for (int j = 0; j < NJ; j++) {
            const int d = j * 16 + d0;
            if constexpr (VEC) {
                const Four<T> t = *reinterpret_cast<const Four<T>*>(p + (d < dk ? d : 0));
#pragma unroll
                for (int i = 0; i < 4; i++) o[j][i] = d < dk ? ld_f32(&t.v[i]) : 0.f;
            } else {
#pragma unroll
                for (int i = 0; i < 4; i++) {
                    const float t = ld_f32(p + min(d + i, dk - 1));
                    o[j][i] = d + i < dk ? t : 0.f;
                }
            }
        }
    };
    auto fetch = [&](int t) {
        t = min(t, end - 1);                               // past the end: a row that exists, never used
        row4(kp + (size_t)t * x.k_stride, kn);
        row4(qp + (size_t)t * x.q_stride, qn);
        vn = ld_f32(vp + (size_t)t * x.v_stride);
    };
#pragma unroll
    for (int j = 0; j < NJ; j++) {
        const int d = j * 16 + d0;
        if constexpr (VEC) {
            const float4 t = *reinterpret_cast<const float4*>(st + (d < dk ? d : 0));
            S[j][0] = t.x; S[j][1] = t.y; S[j][2] = t.z; S[j][3] = t.w;
        } else {
#pragma unroll
            for (int i = 0; i < 4; i++) S[j][i] = st[min(d + i, dk - 1)];
        }
    }
    fetch(begin);
    for (int t = begin; t < end; t++) {
        float k[NJ][4], q[NJ][4];
        const float v = vn;
#pragma unroll
        for (int j = 0; j < NJ; j++)
#pragma unroll
            for (int i = 0; i < 4; i++) { k[j][i] = kn[j][i]; q[j][i] = qn[j][i]; }
        if (t + 1 < end) fetch(t + 1);
        float o = 0.f;
#pragma unroll
        for (int j = 0; j < NJ; j++)
#pragma unroll
            for (int i = 0; i < 4; i++) {
                S[j][i] = __builtin_fmaf(k[j][i], v, g * S[j][i]);
                o = __builtin_fmaf(q[j][i], S[j][i], o);   // (elements past dk: q is zero)
            }
        o += __shfl_xor(o, 1, 64);
        o += __shfl_xor(o, 2, 64);
        if ((lane & 3) == 0 && e < dv) x.y[((size_t)t * H + h) * dv + e] = o;
    }
    if (e >= dv) return;
#pragma unroll
    for (int j = 0; j < NJ; j++) {
        const int d = j * 16 + d0;
        if constexpr (VEC) { if (d < dk) *reinterpret_cast<float4*>(st + d) = make_float4(S[j][0], S[j][1], S[j][2], S[j][3]); }
        else {
#pragma unroll
            for (int i = 0; i < 4; i++) if (d + i < dk) st[d + i] = S[j][i];
        }
    }
}

// ---- chunks --------------------------------------------------------------------------------------------------------------
// E of one chunk.  grid (sequences x chunks, heads, blocks of 64 value elements), four waves: wave w forms the rows
// 16 w .. 16 w + 15 of the block's.  LDS: the decayed values' terms and the keys, both turned so that tokens are contiguous.
__global__ void __launch_bounds__(256)
scan_ends_k(LinearScanArgs x) {
    extern __shared__ __attribute__((aligned(16))) bf16_t ls_lds[];
    bf16_t* const Vt = ls_lds;                             // [3][EB][LCP]
    bf16_t* const Kt = ls_lds + 3 * EB * LCP;              // [dk up to a multiple of 16][LCP]
    const int seq = blockIdx.x / x.n_chunks, chunk = blockIdx.x % x.n_chunks, h = blockIdx.y, e0 = blockIdx.z * EB;
    const int begin = x.cu_rows[seq] + chunk * LC, n = min(LC, x.cu_rows[seq + 1] - begin);
    if (n <= 0) return;
    const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63, r = lane & 15, g = lane >> 4, dk = x.dk, dv = x.dv;
    const int pair = tid & 31, piece = tid >> 5;           // two neighbouring tokens, eight elements of a row
    const int t0 = pair * 2, ta = min(t0, n - 1), tb = min(t0 + 1, n - 1);
    const float dec = x.decay[h];
    const uint4 zero = make_uint4(0, 0, 0, 0);
    union Eight { uint4 u; bf16_t h[8]; };
    {
        const int e = e0 + piece * 8;
        const bf16_t* vp = (const bf16_t*)x.v + (size_t)begin * x.v_stride + (size_t)h * dv + min(e, dv - 8);
        Eight a, b;
        a.u = *reinterpret_cast<const uint4*>(vp + (size_t)ta * x.v_stride);
        b.u = *reinterpret_cast<const uint4*>(vp + (size_t)tb * x.v_stride);
        const float wa = t0 < n && e < dv ? power(dec, n - 1 - t0) : 0.f, wb = t0 + 1 < n && e < dv ? power(dec, n - 2 - t0) : 0.f;
#pragma unroll
        for (int i = 0; i < 8; i++) {
            uint32_t w[3];
            split_two(wa * bf16_to_f32(a.h[i]), wb * bf16_to_f32(b.h[i]), w);
#pragma unroll
            for (int m = 0; m < 3; m++) *reinterpret_cast<uint32_t*>(Vt + (m * EB + piece * 8 + i) * LCP + t0) = w[m];
        }
    }
    const int dkp = (dk + 15) / 16 * 16;
    for (int c = piece; c < dkp / 8; c += 8) {
        const bf16_t* kp = (const bf16_t*)x.k + (size_t)begin * x.k_stride + (size_t)h * dk + (c * 8 < dk ? c * 8 : 0);
        Eight a, b;
        a.u = *reinterpret_cast<const uint4*>(kp + (size_t)ta * x.k_stride);
        b.u = *reinterpret_cast<const uint4*>(kp + (size_t)tb * x.k_stride);
        if (c * 8 >= dk) { a.u = zero; b.u = zero; }
#pragma unroll
        for (int i = 0; i < 8; i++) *reinterpret_cast<uint32_t*>(Kt + (c * 8 + i) * LCP + t0) = (uint32_t)a.h[i] | ((uint32_t)b.h[i] << 16);
    }
    __syncthreads();
    LFrag vf[3][2];
#pragma unroll
    for (int m = 0; m < 3; m++)
#pragma unroll
        for (int s = 0; s < 2; s++) vf[m][s].u = *reinterpret_cast<const uint4*>(Vt + (m * EB + wave * 16 + r) * LCP + s * 32 + g * 8);
    float* out = x.chunks + ((size_t)blockIdx.x * x.H + h) * dv * dk;
    for (int j = 0; j < dkp / 16; j++) {
        ls_f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int s = 0; s < 2; s++) {
            LFrag kf;
            kf.u = *reinterpret_cast<const uint4*>(Kt + (j * 16 + r) * LCP + s * 32 + g * 8);
#pragma unroll
            for (int m = 2; m >= 0; m--) acc = mma(vf[m][s], kf, acc);
        }
        const int d = j * 16 + r, e = e0 + wave * 16 + g * 4;
#pragma unroll
        for (int i = 0; i < 4; i++) if (d < dk && e + i < dv) out[(size_t)(e + i) * dk + d] = acc[i];
    }
}

// The states along a sequence's chunks.  grid (sequences, heads, blocks of 256 quads of S): a thread takes four neighbouring
// elements; AHEAD chunks' E are asked for together.
__global__ void __launch_bounds__(256)
scan_carry_k(LinearScanArgs x) {
    constexpr int AHEAD = 8;
    const int seq = blockIdx.x, h = blockIdx.y, size = x.dv * x.dk, at = (blockIdx.z * 256 + threadIdx.x) * 4;
    const int count = x.cu_rows[seq + 1] - x.cu_rows[seq];
    if (at >= size || count <= 0) return;
    const int chunks = (count + LC - 1) / LC;
    const float dec = x.decay[h], whole = power(dec, LC), last = power(dec, count - (chunks - 1) * LC);
    float4* st = reinterpret_cast<float4*>(x.state + ((size_t)x.slot_ids[seq] * x.H + h) * size + at);
    float* mine = x.chunks + ((size_t)seq * x.n_chunks * x.H + h) * size + at;
    const size_t apart = (size_t)x.H * size;
    float4 s = *st;
    for (int c0 = 0; c0 < chunks; c0 += AHEAD) {
        float4 E[AHEAD];
#pragma unroll
        for (int u = 0; u < AHEAD; u++) E[u] = *reinterpret_cast<const float4*>(mine + (size_t)min(c0 + u, chunks - 1) * apart);
#pragma unroll
        for (int u = 0; u < AHEAD; u++) {
            const int c = c0 + u;
            if (c >= chunks) break;
            *reinterpret_cast<float4*>(mine + (size_t)c * apart) = s;
            const float f = c + 1 < chunks ? whole : last;
            s.x = __builtin_fmaf(f, s.x, E[u].x);
            s.y = __builtin_fmaf(f, s.y, E[u].y);
            s.z = __builtin_fmaf(f, s.z, E[u].z);
            s.w = __builtin_fmaf(f, s.w, E[u].w);
        }
    }
    *st = s;
}

// The outputs of one chunk.  grid (sequences x chunks, heads), four waves.  Wave w first forms the weights of the tokens
// 16 w .. 16 w + 15, turned (keys as rows), so that a lane's four sums are neighbours of one token's row of weights; they meet
// in LDS in three terms.  Then wave w takes the value elements 16 w .. 16 w + 15, + 64, .. of all 64 tokens: its rows of S_0
// come from memory once, asked for before anything else, and are split into their terms in registers.
template <int KS>
__global__ void __launch_bounds__(256)
scan_outputs_k(LinearScanArgs x) {
    extern __shared__ __attribute__((aligned(16))) bf16_t ls_lds[];
    constexpr int KP = KS * 32 + 8;
    bf16_t* const Kr = ls_lds;                             // [LC][KP] keys by rows
    bf16_t* const Qr = Kr + LC * KP;                       // [LC][KP] queries by rows
    bf16_t* const P = Qr + LC * KP;                        // [3][LC tokens][LCP keys]
    bf16_t* const Vt = P + 3 * LC * LCP;                   // [dv up to a multiple of 16][LCP]: values turned
    __shared__ float pow_s[LC + 1];
    const int seq = blockIdx.x / x.n_chunks, chunk = blockIdx.x % x.n_chunks, h = blockIdx.y;
    const int begin = x.cu_rows[seq] + chunk * LC, n = min(LC, x.cu_rows[seq + 1] - begin);
    if (n <= 0) return;
    const int tid = threadIdx.x, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lane = tid & 63, r = lane & 15, g = lane >> 4, dk = x.dk, dv = x.dv;
    const uint4 zero = make_uint4(0, 0, 0, 0);
    const float* const S = x.chunks + ((size_t)blockIdx.x * x.H + h) * dv * dk;
    float4 sr[KS][2];                                      // eight neighbouring elements of row e0 + r of S_0 by k step
    auto rows_of = [&](int e0) {
        const float* p = S + (size_t)min(e0 + r, dv - 1) * dk;
#pragma unroll
        for (int s = 0; s < KS; s++) {
            const int d = s * 32 + g * 8, dc = d < dk ? d : 0;           // (past dk: the queries' elements are zero)
            sr[s][0] = *reinterpret_cast<const float4*>(p + dc);
            sr[s][1] = *reinterpret_cast<const float4*>(p + dc + 4);
        }
    };
    rows_of(min(wave * 16, dv - 1));
    if (tid <= LC) pow_s[tid] = power(x.decay[h], tid);
    {
        const bf16_t* kb = (const bf16_t*)x.k + (size_t)begin * x.k_stride + (size_t)h * dk;
        const bf16_t* qb = (const bf16_t*)x.q + (size_t)begin * x.q_stride + (size_t)h * dk;
#pragma unroll
        for (int i0 = 0; i0 < LC * KS * 4; i0 += 256) {    // (past the chunk's end: its last row; past a row's end: zeros)
            const int i = i0 + tid, t = i / (KS * 4), d = (i - t * (KS * 4)) * 8, dc = d < dk ? d : 0;
            const uint4 kf = *reinterpret_cast<const uint4*>(kb + (size_t)min(t, n - 1) * x.k_stride + dc);
            const uint4 qf = *reinterpret_cast<const uint4*>(qb + (size_t)min(t, n - 1) * x.q_stride + dc);
            *reinterpret_cast<uint4*>(Kr + t * KP + d) = d < dk ? kf : zero;
            *reinterpret_cast<uint4*>(Qr + t * KP + d) = d < dk ? qf : zero;
        }
        const int pair = tid & 31, t0 = pair * 2, ta = min(t0, n - 1), tb = min(t0 + 1, n - 1);
        union Eight { uint4 u; bf16_t h[8]; };
        for (int c = tid >> 5; c < (dv + 15) / 16 * 2; c += 8) {        // values turned, zeros past the chunk's end
            const bf16_t* vp = (const bf16_t*)x.v + (size_t)begin * x.v_stride + (size_t)h * dv + min(c * 8, dv - 8);
            Eight a, b;
            a.u = *reinterpret_cast<const uint4*>(vp + (size_t)ta * x.v_stride);
            b.u = *reinterpret_cast<const uint4*>(vp + (size_t)tb * x.v_stride);
            if (t0 >= n) a.u = zero;
            if (t0 + 1 >= n) b.u = zero;
#pragma unroll
            for (int i = 0; i < 8; i++) *reinterpret_cast<uint32_t*>(Vt + (c * 8 + i) * LCP + t0) = (uint32_t)a.h[i] | ((uint32_t)b.h[i] << 16);
        }
    }
    __syncthreads();
    {
        const int t = wave * 16 + r;
        LFrag qf[KS];
#pragma unroll
        for (int s = 0; s < KS; s++) qf[s].u = *reinterpret_cast<const uint4*>(Qr + t * KP + s * 32 + g * 8);
#pragma unroll
        for (int j = 0; j < 4; j++) {                      // keys 16 j .. 16 j + 15: zeros beyond the wave's own tile
            ls_f32x4 acc = {0.f, 0.f, 0.f, 0.f};
            if (j <= wave) {
#pragma unroll
                for (int s = 0; s < KS; s++) {
                    LFrag kf;
                    kf.u = *reinterpret_cast<const uint4*>(Kr + (j * 16 + r) * KP + s * 32 + g * 8);
                    acc = mma(kf, qf[s], acc);
                }
            }
            float w[4];
#pragma unroll
            for (int i = 0; i < 4; i++) {
                const int s = j * 16 + g * 4 + i;
                w[i] = s <= t ? pow_s[max(t - s, 0)] * acc[i] : 0.f;
            }
            uint32_t lo[3], hi[3];
            split_two(w[0], w[1], lo);
            split_two(w[2], w[3], hi);
#pragma unroll
            for (int m = 0; m < 3; m++) *reinterpret_cast<uint2*>(P + (m * LC + t) * LCP + j * 16 + g * 4) = make_uint2(lo[m], hi[m]);
        }
    }
    __syncthreads();
    const bool quads = dv % 4 == 0;
    for (int e0 = wave * 16; e0 < dv; e0 += 64) {
        LFrag sf[KS][3];
#pragma unroll
        for (int s = 0; s < KS; s++) {
            const float v[8] = {sr[s][0].x, sr[s][0].y, sr[s][0].z, sr[s][0].w, sr[s][1].x, sr[s][1].y, sr[s][1].z, sr[s][1].w};
#pragma unroll
            for (int i = 0; i < 4; i++) {
                uint32_t w[3];
                split_two(v[2 * i], v[2 * i + 1], w);
#pragma unroll
                for (int m = 0; m < 3; m++) sf[s][m].w[i] = w[m];
            }
        }
        if (e0 + 64 < dv) rows_of(e0 + 64);
        LFrag vf[2];
#pragma unroll
        for (int u = 0; u < 2; u++) vf[u].u = *reinterpret_cast<const uint4*>(Vt + (e0 + r) * LCP + u * 32 + g * 8);
#pragma unroll
        for (int tt = 0; tt < 4; tt++) {                   // 16 tokens, a lane one of them
            ls_f32x4 in = {0.f, 0.f, 0.f, 0.f}, in1 = in, own = in;
#pragma unroll
            for (int s = 0; s < KS; s++) {
                LFrag qf;
                qf.u = *reinterpret_cast<const uint4*>(Qr + (tt * 16 + r) * KP + s * 32 + g * 8);
                in1 = mma(sf[s][2], qf, in1);
                in = mma(sf[s][0], qf, in);
                in1 = mma(sf[s][1], qf, in1);
            }
#pragma unroll
            for (int u = 0; u < 2; u++)
                if (u == 0 || tt >= 2) {                   // (the lower half's tokens see no key of the upper half)
#pragma unroll
                    for (int m = 2; m >= 0; m--) {
                        LFrag pf;
                        pf.u = *reinterpret_cast<const uint4*>(P + (m * LC + tt * 16 + r) * LCP + u * 32 + g * 8);
                        own = mma(vf[u], pf, own);
                    }
                }
            in = in + in1;
            const int t = tt * 16 + r, e = e0 + g * 4;
            const float since = pow_s[t + 1];
            if (t < n) {
                float* yr = x.y + ((size_t)(begin + t) * x.H + h) * dv;
                if (quads) {
                    if (e < dv)
                        *reinterpret_cast<float4*>(yr + e) = make_float4(__builtin_fmaf(since, in[0], own[0]), __builtin_fmaf(since, in[1], own[1]),
                                                                         __builtin_fmaf(since, in[2], own[2]), __builtin_fmaf(since, in[3], own[3]));
                } else {
#pragma unroll
                    for (int i = 0; i < 4; i++) if (e + i < dv) yr[e + i] = __builtin_fmaf(since, in[i], own[i]);
                }
            }
        }
    }
}

static size_t ls_align(size_t n) { return (n + 255) / 256 * 256; }

extern "C" long tp_linear_scan_workspace_bytes(int n_seq, int n_chunks, int H, int dk, int dv) {
    const size_t el = (size_t)n_seq * n_chunks * H * dk * dv;
    return (long)ls_align(el * sizeof(float));
}

// q, k [M, H dk], v [M, H dv] as views of wider rows of one dtype; decay float32 [H]; state [slots, H, dv, dk] float32, left
// updated; y float32 [M, H dv].  n_chunks > 0: bfloat16 steps in chunks of 64 tokens, that many covering the longest sequence.
extern "C" int tp_linear_scan(const void* q, long q_stride, const void* k, long k_stride, const void* v, long v_stride, int dtype,
                              const float* decay, float* state, const int* slot_ids, const int* cu_rows, float* y, int n_seq, int H,
                              int dk, int dv, int n_chunks, void* workspace, long workspace_bytes, void* stream) {
    TP_REQUIRE(n_seq > 0 && H > 0 && dk > 0 && dv > 0, "linear_scan: empty shape sequences=%d heads=%d key=%d value=%d", n_seq, H, dk, dv);
    TP_REQUIRE(dk <= 256 && dv <= 256, "linear_scan: heads of %d x %d exceed 256 x 256", dk, dv);
    TP_REQUIRE(H <= 65535, "linear_scan: %d heads exceed one launch", H);
    TP_REQUIRE(q && k && v && decay && state && slot_ids && cu_rows && y, "linear_scan: null operand");
    TP_REQUIRE(dtype == TP_BF16 || dtype == TP_F32, "linear_scan: unknown dtype %d", dtype);
    hipStream_t s = (hipStream_t)stream;
    LinearScanArgs x{q, q_stride, k, k_stride, v, v_stride, decay, state, slot_ids, cu_rows, y, n_seq, H, dk, dv, n_chunks, nullptr};
    if (n_chunks > 0) {
        TP_REQUIRE(dtype == TP_BF16 && dk % 8 == 0 && dv % 8 == 0 && q_stride % 8 == 0 && k_stride % 8 == 0 && v_stride % 8 == 0 &&
                   (uintptr_t)q % 16 == 0 && (uintptr_t)k % 16 == 0 && (uintptr_t)v % 16 == 0, "linear_scan: chunks need bfloat16 rows of whole 16-byte pieces");
        TP_REQUIRE((long)n_seq * n_chunks <= 0x7fffffffL, "linear_scan: %d chunks of %d sequences exceed one launch", n_chunks, n_seq);
        TP_REQUIRE(workspace && (uintptr_t)workspace % 16 == 0 && workspace_bytes >= tp_linear_scan_workspace_bytes(n_seq, n_chunks, H, dk, dv),
                   "linear_scan: a workspace of %ld bytes is too small", workspace_bytes);
        x.chunks = (float*)workspace;
        const int units = n_seq * n_chunks, ks = tp_cdiv(dk, 32), ksr = ks <= 4 ? ks : (ks <= 6 ? 6 : 8);
        const size_t lds_ends = (size_t)(3 * EB + (dk + 15) / 16 * 16) * LCP * sizeof(bf16_t);
        const size_t lds_out = ((size_t)2 * LC * (ksr * 32 + 8) + 3 * LC * LCP + (size_t)((dv + 15) / 16 * 16) * LCP) * sizeof(bf16_t);
        auto room = [](const void* kernel, size_t bytes) {       // more LDS than a kernel gets without asking
            return bytes <= 65536 || hipFuncSetAttribute(kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)bytes) == hipSuccess;
        };
        TP_REQUIRE(room((const void*)scan_ends_k, lds_ends), "linear_scan: cannot reserve %zu bytes of LDS", lds_ends);
        scan_ends_k<<<dim3(units, H, tp_cdiv(dv, EB)), 256, lds_ends, s>>>(x);
        scan_carry_k<<<dim3(n_seq, H, tp_cdiv((long)dv * dk, 1024)), 256, 0, s>>>(x);
#define TP_SCAN_OUT(KS) do { \
            TP_REQUIRE(room((const void*)scan_outputs_k<KS>, lds_out), "linear_scan: cannot reserve %zu bytes of LDS", lds_out); \
            scan_outputs_k<KS><<<dim3(units, H), 256, lds_out, s>>>(x); } while (0)
        switch (ksr) {
            case 1: TP_SCAN_OUT(1); break;
            case 2: TP_SCAN_OUT(2); break;
            case 3: TP_SCAN_OUT(3); break;
            case 4: TP_SCAN_OUT(4); break;
            case 6: TP_SCAN_OUT(6); break;
            default: TP_SCAN_OUT(8); break;
        }
#undef TP_SCAN_OUT
        return tp_check_launch("linear_scan (chunks)");
    }
    const long el = dtype == TP_BF16 ? 2 : 4;
    const bool vec = dk % 4 == 0 && q_stride % 4 == 0 && k_stride % 4 == 0 && (uintptr_t)q % (4 * el) == 0 && (uintptr_t)k % (4 * el) == 0;
    dim3 grid(n_seq, H, tp_cdiv(dv, 16));
#define TP_SCAN_ROWS(NJ) do { \
        if (dtype == TP_BF16) { if (vec) scan_rows_k<bf16_t, NJ, true><<<grid, 64, 0, s>>>(x); else scan_rows_k<bf16_t, NJ, false><<<grid, 64, 0, s>>>(x); } \
        else { if (vec) scan_rows_k<float, NJ, true><<<grid, 64, 0, s>>>(x); else scan_rows_k<float, NJ, false><<<grid, 64, 0, s>>>(x); } } while (0)
    if (dk <= 64) TP_SCAN_ROWS(4);
    else if (dk <= 128) TP_SCAN_ROWS(8);
    else TP_SCAN_ROWS(16);
#undef TP_SCAN_ROWS
    return tp_check_launch("linear_scan");
}
