// Recurrent time mixing with a token shift: what several projections read are mixes of a token's row and
// the row of the token before it, and per head a matrix of state S [d, d] (float32) decays by a number of
// its own a key channel and token:
//     in_s = h + (h_before - h) mu_s                                   (h_before 0 for the first token)
//     w = exp(-exp(z + w0)),   o = (S + diag(u) k v^T)^T r,   S <- diag(w) S + k v^T
//   token_mix           the mixes in_0 .. in_(S-1) of a step's rows
//   time_mix_prepare    the inputs of illm_gated_scan (rule 2: o from the state before the token, with
//                       beta = sum u r k as the weight of v)
//   time_mix_chunks     long steps, chunks of TM_CHUNK tokens in parallel (below)
// (single tokens: illm_time_mix_step in fixed_decay.hip).  Everything but the stored projections is
// float32.  A sequence's rows in a step are consecutive.
#include <math.h>

#include "api.h"
#include "common.h"

// ---------------------------------------------------------------- token shift
// grid (rows, ceil(E / (256 VEC))).  out [S][T][E].  The row before a step's first row of a sequence comes
// from tail [slots][E]; a step of single tokens moves it on in the same launch (`update_tail`).
template <int VEC>
__global__ void __launch_bounds__(256)
token_mix_kernel(const void* __restrict__ X, int dt, const float* __restrict__ mu, int S, void* __restrict__ tail,
                 const int32_t* __restrict__ row_slot, void* __restrict__ out, int out_dt, int T, int E,
                 int update_tail) {
    const int r = blockIdx.x, c = blockIdx.y * 256 + threadIdx.x;
    if (VEC * c >= E) return;
    const int slot = row_slot[r];
    const bool own = r > 0 && row_slot[r - 1] == slot;
    if (VEC == 4) {
        const size_t n4 = E / 4;
        const float4 x = ld_f4(X, dt, r * n4 + c);
        const float4 p = own ? ld_f4(X, dt, (r - 1) * n4 + c) : ld_f4(tail, dt, slot * n4 + c);
        const float4 d = make_float4(p.x - x.x, p.y - x.y, p.z - x.z, p.w - x.w);
        for (int s = 0; s < S; ++s) {
            const float4 m = ((const float4*)mu)[s * n4 + c];
            st_f4(out, out_dt, ((size_t)s * T + r) * n4 + c,
                  make_float4(fmaf(d.x, m.x, x.x), fmaf(d.y, m.y, x.y), fmaf(d.z, m.z, x.z), fmaf(d.w, m.w, x.w)));
        }
        if (update_tail) st_f4(tail, dt, slot * n4 + c, x);
        return;
    }
    const float x = ld_f(X, dt, (size_t)r * E + c);
    const float p = own ? ld_f(X, dt, (size_t)(r - 1) * E + c) : ld_f(tail, dt, (size_t)slot * E + c);
    for (int s = 0; s < S; ++s) st_f(out, out_dt, ((size_t)s * T + r) * E + c, fmaf(p - x, mu[(size_t)s * E + c], x));
    if (update_tail) st_f(tail, dt, (size_t)slot * E + c, x);
}

extern "C" int illm_token_mix(const void* X, int dt, const float* mu, int S, void* tail, const int32_t* row_slot,
                              void* out, int out_dt, int T, int E, int update_tail, void* stream) {
    if (T < 0 || E <= 0 || S <= 0 || !illm_dtype_ok(dt) || !illm_dtype_ok(out_dt) || (E + 255) / 256 > 65535)
        return ILLM_ERR_ARG;
    if (T == 0) return ILLM_OK;
    if (E % 4 == 0)
        hipLaunchKernelGGL(token_mix_kernel<4>, dim3(T, (E / 4 + 255) / 256), dim3(256), 0, (hipStream_t)stream, X, dt,
                           mu, S, tail, row_slot, out, out_dt, T, E, update_tail);
    else
        hipLaunchKernelGGL(token_mix_kernel<1>, dim3(T, (E + 255) / 256), dim3(256), 0, (hipStream_t)stream, X, dt, mu,
                           S, tail, row_slot, out, out_dt, T, E, update_tail);
    return illm_launch_status();
}

// ---------------------------------------------------------------- inputs of the scan
// grid (rows, ceil(H / 4)); a wave takes a head, lanes over its d channels (d <= 256).  r, k, v rows of
// `stride` numbers, Z float32 [T, H d].
#define TM_VEC 4
__global__ void __launch_bounds__(256)
time_mix_prepare_kernel(const void* __restrict__ R, const void* __restrict__ K, const void* __restrict__ V, int dt,
                        int stride, const float* __restrict__ Z, const float* __restrict__ w0,
                        const float* __restrict__ bonus, float* __restrict__ qn, float* __restrict__ kn,
                        float* __restrict__ vv, float* __restrict__ beta, float* __restrict__ dec, int H, int d) {
    const size_t t = blockIdx.x, u0 = t * stride;
    const int h = blockIdx.y * 4 + wave_index(), lane = threadIdx.x & 63;
    if (h >= H) return;
    float sum = 0.f;
#pragma unroll
    for (int e = 0; e < TM_VEC; ++e) {
        const int i = lane + 64 * e, c = h * d + i;
        if (i >= d) continue;
        const size_t at = t * H * d + c;
        const float r = ld_f(R, dt, u0 + c), k = ld_f(K, dt, u0 + c);
        sum = fmaf(r * bonus[c], k, sum);
        qn[at] = r;
        kn[at] = k;
        vv[at] = ld_f(V, dt, u0 + c);
        dec[at] = expf(-expf(Z[at] + w0[c]));
    }
    sum = wave_sum(sum);
    if (lane == 0) beta[t * H + h] = sum;
}

extern "C" int illm_time_mix_prepare(const void* R, const void* K, const void* V, int dt, int stride, const float* Z,
                                     const float* w0, const float* bonus, float* qn, float* kn, float* vv, float* beta,
                                     float* dec, int T, int H, int d, void* stream) {
    if (T < 0 || H <= 0 || d <= 0 || d > 64 * TM_VEC || !illm_dtype_ok(dt) || stride < H * d || (H + 3) / 4 > 65535)
        return ILLM_ERR_ARG;
    if (T == 0) return ILLM_OK;
    hipLaunchKernelGGL(time_mix_prepare_kernel, dim3(T, (H + 3) / 4), dim3(256), 0, (hipStream_t)stream, R, K, V, dt,
                       stride, Z, w0, bonus, qn, kn, vv, beta, dec, H, d);
    return illm_launch_status();
}

// ---------------------------------------------------------------- long steps in chunks
// A step's rows of a sequence in chunks of TM_CHUNK tokens, each in sub-blocks of TM_SUB:
//   decay_sums   per channel the sums of log2 w within a sub-block, up to and with each token: L
//   chunk_sums   per (chunk, head) sum_j diag(w after j) k_j v_j^T, the chunk's part of the state, and the
//                chunk's whole decays
//   chunk_carry  per head, chunk after chunk: the state at every chunk's start (in place of the parts) and
//                the sequence's last state back into the slot
//   chunk_rows   per (chunk, head), a wave a sub-block: the rows from the chunk's start state, from the sub-
//                blocks before theirs and from their own
// Every decay that is applied is exp2 of a sum that is never positive: a sum within a sub-block counts from
// its token or up to it, whole sub-blocks between are factors of their own.  Nothing is divided by a decay, so
// a channel may forget everything within a token.  A log2 of a decay is held above TM_FLOOR: what is left of a
// number after one such token is below 2^-57 of it either way, and the sums keep their digits.
// Products are MFMA 16x16x4 and 32x32x2 with float32 operands, products and sums.  Chunk c of sequence b lies
// at place cu[b] / TM_CHUNK + b + c.  Head sizes up to 128 in steps of 4, filled up with zeros.
#define TM_CHUNK 64
#define TM_SUB 16
#define TM_FLOOR -58.0f
#define LOG2_E 1.44269504088896340736f
typedef float tm_f32x4_t __attribute__((ext_vector_type(4)));
typedef float tm_f32x16_t __attribute__((ext_vector_type(16)));

__device__ __forceinline__ float tm_exp2(float x) { return __builtin_amdgcn_exp2f(x); }

// grid (ceil(n / 256), sub-blocks, sequences); a thread a channel of a sub-block.  Z [T, n] -> L [T, n].
__global__ void __launch_bounds__(256)
time_mix_decay_sums_kernel(const float* __restrict__ Z, const float* __restrict__ w0, float* __restrict__ L,
                           const int32_t* __restrict__ cu, int n) {
    const int b = blockIdx.z, c = blockIdx.x * 256 + threadIdx.x;
    const int r0 = cu[b], len = cu[b + 1] - r0, t0 = blockIdx.y * TM_SUB;
    if (t0 >= len || c >= n) return;
    const int m = min(TM_SUB, len - t0);
    const size_t at = (size_t)(r0 + t0) * n + c;
    const float off = w0[c];
    float z[TM_SUB];
#pragma unroll
    for (int t = 0; t < TM_SUB; ++t) z[t] = Z[at + (size_t)min(t, m - 1) * n];
    float sum = 0.f;
#pragma unroll
    for (int t = 0; t < TM_SUB; ++t) {
        if (t >= m) continue;
        sum += fmaxf(-expf(z[t] + off) * LOG2_E, TM_FLOOR);
        L[at + (size_t)t * n] = sum;
    }
}

// grid (chunks, H, sequences); 256 threads.  part [places][H][d][d], whole [places][H][d].
template <int DT, int KT>
__global__ void __launch_bounds__(256)
time_mix_chunk_sums_kernel(const void* __restrict__ K, const void* __restrict__ V, int stride,
                           const float* __restrict__ L, float* __restrict__ part, float* __restrict__ whole,
                           const int32_t* __restrict__ cu, int H, int d) {
    constexpr int DP = 32 * KT, NT = (KT * KT + 3) / 4, QUADS = DP / 4, ROWS = 256 / QUADS;
    __shared__ float ks[TM_CHUNK * DP];
    __shared__ float vs[TM_CHUNK * DP];
    const int b = blockIdx.z, h = blockIdx.y, c = blockIdx.x, tid = threadIdx.x;
    const int r0 = cu[b], n = cu[b + 1] - r0, t0 = c * TM_CHUNK;
    if (t0 >= n) return;                                // the whole block
    const int nc = min(TM_CHUNK, n - t0), ld = H * d;
    const size_t place = (size_t)(r0 / TM_CHUNK + b + c) * H + h;
    {
        // a thread's rows all have the same four channels: the sub-blocks' whole sums are read once
        const int i4 = 4 * (tid % QUADS);
        const bool in = i4 < d;
        const float* Lc = L + (size_t)(r0 + t0) * ld + (size_t)h * d + (in ? i4 : 0);
        float4 tot[TM_CHUNK / TM_SUB], after[TM_CHUNK / TM_SUB];
#pragma unroll
        for (int s = 0; s < TM_CHUNK / TM_SUB; ++s) {
            tot[s] = make_float4(0.f, 0.f, 0.f, 0.f);
            if (TM_SUB * s < nc) tot[s] = *(const float4*)(Lc + (size_t)min(TM_SUB * s + TM_SUB - 1, nc - 1) * ld);
        }
        float4 run = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
        for (int s = TM_CHUNK / TM_SUB - 1; s >= 0; --s) {
            after[s] = run;                             // log2 of the decays of the sub-blocks behind s
            run.x += tot[s].x; run.y += tot[s].y; run.z += tot[s].z; run.w += tot[s].w;
        }
        if (tid < QUADS && in)
            *(float4*)(whole + place * d + i4) = make_float4(tm_exp2(run.x), tm_exp2(run.y), tm_exp2(run.z), tm_exp2(run.w));
#pragma unroll
        for (int s = 0; s < TM_CHUNK / TM_SUB; ++s)
            for (int x = tid / QUADS; x < TM_SUB; x += ROWS) {
                const int row = TM_SUB * s + x;
                float4 k = make_float4(0.f, 0.f, 0.f, 0.f), v = k;
                if (row < nc && in) {
                    const size_t at = ((size_t)(r0 + t0 + row) * stride + (size_t)h * d + i4) / 4;
                    const float4 l = *(const float4*)(Lc + (size_t)row * ld);
                    k = ld_f4(K, DT, at);
                    v = ld_f4(V, DT, at);
                    k.x *= tm_exp2((tot[s].x - l.x) + after[s].x); k.y *= tm_exp2((tot[s].y - l.y) + after[s].y);
                    k.z *= tm_exp2((tot[s].z - l.z) + after[s].z); k.w *= tm_exp2((tot[s].w - l.w) + after[s].w);
                }
                *(float4*)(ks + row * DP + i4) = k;
                *(float4*)(vs + row * DP + i4) = v;
            }
    }
    __syncthreads();
    const int lane = tid & 63, w = wave_index(), col = lane & 31, half = lane >> 5;
    float* dst = part + place * d * d;
#pragma unroll
    for (int x = 0; x < NT; ++x) {
        const int tile = w + 4 * x;
        if (tile >= KT * KT) continue;
        const int m0 = 32 * (tile / KT), n0 = 32 * (tile % KT);
        tm_f32x16_t acc;
#pragma unroll
        for (int v = 0; v < 16; ++v) acc[v] = 0.f;
#pragma unroll 8
        for (int s2 = 0; s2 < TM_CHUNK / 2; ++s2)
            acc = __builtin_amdgcn_mfma_f32_32x32x2f32(ks[(2 * s2 + half) * DP + m0 + col],
                                                       vs[(2 * s2 + half) * DP + n0 + col], acc, 0, 0, 0);
#pragma unroll
        for (int v = 0; v < 16; ++v) {
            const int m = m0 + 8 * (v >> 2) + 4 * half + (v & 3), nn = n0 + col;
            if (m < d && nn < d) dst[(size_t)m * d + nn] = acc[v];
        }
    }
}

// grid (ceil(d d / 1024), H, sequences); 256 threads, 4 neighbouring numbers of a row each.
#define TM_AHEAD 8
__global__ void __launch_bounds__(256)
time_mix_chunk_carry_kernel(float* __restrict__ part, const float* __restrict__ whole, float* __restrict__ state,
                            const int32_t* __restrict__ cu, const int32_t* __restrict__ seq_slot, int H, int d) {
    const int b = blockIdx.z, h = blockIdx.y, i4 = blockIdx.x * 256 + threadIdx.x;
    const int r0 = cu[b], n = cu[b + 1] - r0, n4 = d * d / 4;
    if (n <= 0 || i4 >= n4) return;
    const int chunks = (n + TM_CHUNK - 1) / TM_CHUNK;
    const size_t place = (size_t)(r0 / TM_CHUNK + b) * H + h;
    float4* sp = (float4*)(state + ((size_t)seq_slot[b] * H + h) * d * d) + i4;
    float4* pp = (float4*)(part + place * d * d) + i4;
    const float* wp = whole + place * d + 4 * i4 / d;
    const size_t step = (size_t)H * n4, wstep = (size_t)H * d;
    float4 S = *sp;
    for (int c0 = 0; c0 < chunks; c0 += TM_AHEAD) {
        float4 add[TM_AHEAD];
        float f[TM_AHEAD];
#pragma unroll
        for (int x = 0; x < TM_AHEAD; ++x) {
            const int c = min(c0 + x, chunks - 1);
            add[x] = pp[(size_t)c * step];
            f[x] = wp[(size_t)c * wstep];
        }
#pragma unroll
        for (int x = 0; x < TM_AHEAD; ++x) {
            if (c0 + x >= chunks) continue;
            pp[(size_t)(c0 + x) * step] = S;
            S.x = fmaf(f[x], S.x, add[x].x); S.y = fmaf(f[x], S.y, add[x].y);
            S.z = fmaf(f[x], S.z, add[x].z); S.w = fmaf(f[x], S.w, add[x].w);
        }
    }
    *sp = S;
}

// four neighbouring numbers in LDS of the storage type
__device__ __forceinline__ float4 tm_lds4(const bf16_t* p) {
    const uint2 u = *(const uint2*)p;
    return make_float4(__uint_as_float(u.x << 16), __uint_as_float(u.x & 0xffff0000u), __uint_as_float(u.y << 16),
                       __uint_as_float(u.y & 0xffff0000u));
}
__device__ __forceinline__ float4 tm_lds4(const float* p) { return *(const float4*)p; }
__device__ __forceinline__ float tm_lds1(const bf16_t* p) { return bf16_to_f32(*p); }
__device__ __forceinline__ float tm_lds1(const float* p) { return *p; }

template <int DT> struct TmStored;
template <> struct TmStored<ILLM_BF16> { typedef bf16_t type; };
template <> struct TmStored<ILLM_F32> { typedef float type; };

template <int DT, int KS>
constexpr size_t time_mix_rows_lds() {
    return (size_t)TM_CHUNK * ((16 * KS + 4) * 4 + (16 * KS + 16 / sizeof(typename TmStored<DT>::type)) *
                                                       sizeof(typename TmStored<DT>::type) * 2);
}

// grid (chunks, H, sequences); 256 threads, dynamic LDS.  Wave a takes the chunk's tokens 16 a .. 16 a + 15; a
// lane (t = lane % 16, g = lane / 16) holds token t's channels 16 s + 4 g .. + 3.  All products are kept transposed
// (a column is a token): scores^T = K . R^T leaves keys 4 g .. 4 g + 3 of token t in a lane, which are the second
// operand of o^T += V^T . scores^T as they stand.  Within the wave's own sub-block a pair's decays differ from pair
// to pair: those scores are sums on the vector units, a lane over its channels for all 16 keys.
template <int DT, int KS>
__global__ void __launch_bounds__(256)
time_mix_chunk_rows_kernel(const void* __restrict__ R, const void* __restrict__ K, const void* __restrict__ V,
                           int stride, const float* __restrict__ L, const float* __restrict__ bonus,
                           const float* __restrict__ part, const int32_t* __restrict__ cu, float* __restrict__ o,
                           int H, int d) {
    typedef typename TmStored<DT>::type T;
    constexpr int DP = 16 * KS, LLD = DP + 4, SLD = DP + 16 / (int)sizeof(T);
    extern __shared__ __attribute__((aligned(16))) char tm_smem[];
    float* ls = (float*)tm_smem;                         // [64][LLD]
    T* ks = (T*)(ls + TM_CHUNK * LLD);                   // [64][SLD]
    T* vs = ks + TM_CHUNK * SLD;                         // [64][SLD]
    const int b = blockIdx.z, h = blockIdx.y, c = blockIdx.x, tid = threadIdx.x;
    const int r0 = cu[b], n = cu[b + 1] - r0, t0 = c * TM_CHUNK;
    if (t0 >= n) return;                                 // the whole block
    const int nc = min(TM_CHUNK, n - t0), ld = H * d;
    for (int e = tid; e < TM_CHUNK * (DP / 4); e += 256) {
        const int row = e / (DP / 4), i4 = 4 * (e % (DP / 4));
        const bool ok = row < nc && i4 < d;
        const size_t at = (size_t)(r0 + t0 + (ok ? row : 0)) * stride + (size_t)h * d + (ok ? i4 : 0);
        *(float4*)(ls + row * LLD + i4) =
            ok ? *(const float4*)(L + (size_t)(r0 + t0 + row) * ld + (size_t)h * d + i4) : make_float4(0.f, 0.f, 0.f, 0.f);
        if (DT == ILLM_BF16) {
            const uint2 zero = make_uint2(0u, 0u);
            *(uint2*)((bf16_t*)ks + row * SLD + i4) = ok ? *(const uint2*)((const bf16_t*)K + at) : zero;
            *(uint2*)((bf16_t*)vs + row * SLD + i4) = ok ? *(const uint2*)((const bf16_t*)V + at) : zero;
        } else {
            const float4 zero = make_float4(0.f, 0.f, 0.f, 0.f);
            *(float4*)((float*)ks + row * SLD + i4) = ok ? *(const float4*)((const float*)K + at) : zero;
            *(float4*)((float*)vs + row * SLD + i4) = ok ? *(const float4*)((const float*)V + at) : zero;
        }
    }
    __syncthreads();
    const int a = wave_index(), lane = tid & 63, tl = lane & 15, g = lane >> 4, t = TM_SUB * a + tl;
    if (TM_SUB * a >= nc) return;                        // (no barrier follows)
    float rr[KS][4], es[KS][4];                          // r, and log2 of the decays before the token in its sub-block
    float own = 0.f;                                     // sum u r k over the lane's channels
    {
        const size_t at = (size_t)(r0 + t0 + min(t, nc - 1)) * stride + (size_t)h * d + 4 * g;
#pragma unroll
        for (int s = 0; s < KS; ++s) {
            const int i4 = 16 * s + 4 * g;
            float4 x = make_float4(0.f, 0.f, 0.f, 0.f), u = x, l = x;
            if (i4 < d) { x = ld_f4(R, DT, (at + 16 * s) / 4); u = *(const float4*)(bonus + (size_t)h * d + i4); }
            const float4 k = tm_lds4(ks + t * SLD + i4);
            if (tl > 0) l = *(const float4*)(ls + (t - 1) * LLD + i4);
            rr[s][0] = x.x; rr[s][1] = x.y; rr[s][2] = x.z; rr[s][3] = x.w;
            es[s][0] = l.x; es[s][1] = l.y; es[s][2] = l.z; es[s][3] = l.w;
            own = fmaf(x.x * u.x, k.x, own); own = fmaf(x.y * u.y, k.y, own);
            own = fmaf(x.z * u.z, k.z, own); own = fmaf(x.w * u.w, k.w, own);
        }
    }
    own += __shfl_xor(own, 16, ILLM_WAVE);
    own += __shfl_xor(own, 32, ILLM_WAVE);
    tm_f32x4_t acc[KS];
#pragma unroll
    for (int m = 0; m < KS; ++m) acc[m] = (tm_f32x4_t){0.f, 0.f, 0.f, 0.f};
    // o^T += V^T of sub-block x . p, p[v] the weight of key 4 g + v for token t
    auto add_values = [&](int x, const tm_f32x4_t p) __attribute__((always_inline)) {
#pragma unroll
        for (int v = 0; v < 4; ++v) {
            const T* vr = vs + (TM_SUB * x + 4 * g + v) * SLD + tl;
#pragma unroll
            for (int m = 0; m < KS; ++m)
                acc[m] = __builtin_amdgcn_mfma_f32_16x16x4f32(tm_lds1(vr + 16 * m), p[v], acc[m], 0, 0, 0);
        }
    };
    {
        float sc[TM_SUB];
#pragma unroll
        for (int j = 0; j < TM_SUB; ++j) {
            const T* kr = ks + (TM_SUB * a + j) * SLD + 4 * g;
            const float* lr = ls + (TM_SUB * a + j) * LLD + 4 * g;
            float s0 = 0.f, s1 = 0.f;
#pragma unroll
            for (int s = 0; s < KS; ++s) {
                const float4 k = tm_lds4(kr + 16 * s), l = *(const float4*)(lr + 16 * s);
                // (keys at or after the token are left out below; their exponents are only kept finite)
                s0 = fmaf(rr[s][0] * k.x, tm_exp2(fminf(es[s][0] - l.x, 0.f)), s0);
                s1 = fmaf(rr[s][1] * k.y, tm_exp2(fminf(es[s][1] - l.y, 0.f)), s1);
                s0 = fmaf(rr[s][2] * k.z, tm_exp2(fminf(es[s][2] - l.z, 0.f)), s0);
                s1 = fmaf(rr[s][3] * k.w, tm_exp2(fminf(es[s][3] - l.w, 0.f)), s1);
            }
            sc[j] = s0 + s1;
        }
        // the sums over the four lanes of a token, each of which keeps four keys
        float h8[8];
        tm_f32x4_t p;
#pragma unroll
        for (int j = 0; j < 8; ++j) {
            const float keep = g & 2 ? sc[8 + j] : sc[j], send = g & 2 ? sc[j] : sc[8 + j];
            h8[j] = keep + __shfl_xor(send, 32, ILLM_WAVE);
        }
#pragma unroll
        for (int v = 0; v < 4; ++v) {
            const float keep = g & 1 ? h8[4 + v] : h8[v], send = g & 1 ? h8[v] : h8[4 + v];
            const float sum = keep + __shfl_xor(send, 16, ILLM_WAVE);
            const int j = 4 * g + v;
            p[v] = j < tl ? sum : j == tl ? own : 0.f;
        }
        add_values(a, p);
    }
#pragma unroll
    for (int s = 0; s < KS; ++s)
#pragma unroll
        for (int e = 0; e < 4; ++e) rr[s][e] *= tm_exp2(es[s][e]);       // from here on: decayed since the sub-block's start
    for (int x = a - 1; x >= 0; --x) {
        const T* kr = ks + (TM_SUB * x + tl) * SLD + 4 * g;
        const float* lr = ls + (TM_SUB * x + tl) * LLD + 4 * g;
        const float* le = ls + (TM_SUB * x + TM_SUB - 1) * LLD + 4 * g;
        tm_f32x4_t sc = (tm_f32x4_t){0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int s = 0; s < KS; ++s) {
            const float4 k = tm_lds4(kr + 16 * s), l = *(const float4*)(lr + 16 * s), q = *(const float4*)(le + 16 * s);
            sc = __builtin_amdgcn_mfma_f32_16x16x4f32(k.x * tm_exp2(q.x - l.x), rr[s][0], sc, 0, 0, 0);
            sc = __builtin_amdgcn_mfma_f32_16x16x4f32(k.y * tm_exp2(q.y - l.y), rr[s][1], sc, 0, 0, 0);
            sc = __builtin_amdgcn_mfma_f32_16x16x4f32(k.z * tm_exp2(q.z - l.z), rr[s][2], sc, 0, 0, 0);
            sc = __builtin_amdgcn_mfma_f32_16x16x4f32(k.w * tm_exp2(q.w - l.w), rr[s][3], sc, 0, 0, 0);
            rr[s][0] *= tm_exp2(q.x); rr[s][1] *= tm_exp2(q.y); rr[s][2] *= tm_exp2(q.z); rr[s][3] *= tm_exp2(q.w);
        }
        add_values(x, sc);
    }
    // from the chunk's start state (rows beyond d meet zeros of r, columns beyond it are not stored)
    const float* S = part + ((size_t)(r0 / TM_CHUNK + b + c) * H + h) * d * d;
#pragma unroll
    for (int m = 0; m < KS; ++m) {
        const float* Sc = S + min(16 * m + tl, d - 1);
        float av[4 * KS];
#pragma unroll
        for (int s = 0; s < KS; ++s)
#pragma unroll
            for (int e = 0; e < 4; ++e) av[4 * s + e] = Sc[(size_t)min(16 * s + 4 * g + e, d - 1) * d];
#pragma unroll
        for (int s = 0; s < KS; ++s)
#pragma unroll
            for (int e = 0; e < 4; ++e)
                acc[m] = __builtin_amdgcn_mfma_f32_16x16x4f32(av[4 * s + e], rr[s][e], acc[m], 0, 0, 0);
    }
    if (t >= nc) return;
    float* op = o + ((size_t)(r0 + t0 + t) * H + h) * d;
#pragma unroll
    for (int m = 0; m < KS; ++m) {
        const int i4 = 16 * m + 4 * g;
        if (i4 < d) *(float4*)(op + i4) = make_float4(acc[m][0], acc[m][1], acc[m][2], acc[m][3]);
    }
}

template <int DT, int KS>
static int time_mix_rows_launch(const void* R, const void* K, const void* V, int stride, const float* L,
                                const float* bonus, const float* part, const int32_t* cu, float* o, int chunks,
                                int n_seqs, int H, int d, hipStream_t st) {
    constexpr size_t lds = time_mix_rows_lds<DT, KS>();
    if (lds > 48 * 1024 &&
        hipFuncSetAttribute((const void*)time_mix_chunk_rows_kernel<DT, KS>, hipFuncAttributeMaxDynamicSharedMemorySize,
                            (int)lds) != hipSuccess)
        return ILLM_ERR_LAUNCH;
    hipLaunchKernelGGL((time_mix_chunk_rows_kernel<DT, KS>), dim3(chunks, H, n_seqs), dim3(256), lds, st, R, K, V,
                       stride, L, bonus, part, cu, o, H, d);
    return illm_launch_status();
}

template <int DT>
static int time_mix_chunks_launch(const void* R, const void* K, const void* V, int stride, const float* L,
                                  const float* bonus, float* state, float* part, float* whole, const int32_t* cu,
                                  const int32_t* seq_slot, float* o, int n_seqs, int max_rows, int H, int d,
                                  hipStream_t st) {
    const int chunks = (max_rows + TM_CHUNK - 1) / TM_CHUNK, kt = (d + 31) / 32;
    const dim3 grid(chunks, H, n_seqs);
#define SUMS(KT_)                                                                                       \
    hipLaunchKernelGGL((time_mix_chunk_sums_kernel<DT, KT_>), grid, dim3(256), 0, st, K, V, stride, L, part, whole, \
                       cu, H, d)
    if (kt <= 1) SUMS(1);
    else if (kt <= 2) SUMS(2);
    else SUMS(4);
#undef SUMS
    hipLaunchKernelGGL(time_mix_chunk_carry_kernel, dim3((d * d / 4 + 255) / 256, H, n_seqs), dim3(256), 0, st, part,
                       whole, state, cu, seq_slot, H, d);
    if (hipGetLastError() != hipSuccess) return ILLM_ERR_LAUNCH;
    if (kt <= 1)
        return time_mix_rows_launch<DT, 2>(R, K, V, stride, L, bonus, part, cu, o, chunks, n_seqs, H, d, st);
    if (kt <= 2)
        return time_mix_rows_launch<DT, 4>(R, K, V, stride, L, bonus, part, cu, o, chunks, n_seqs, H, d, st);
    return time_mix_rows_launch<DT, 8>(R, K, V, stride, L, bonus, part, cu, o, chunks, n_seqs, H, d, st);
}

extern "C" int illm_time_mix_chunk(void) { return TM_CHUNK; }

// L: T H d floats of scratch; part: (T / TM_CHUNK + n_seqs + 1) H d d floats; whole: as many H d floats.
extern "C" int illm_time_mix_chunks(const void* R, const void* K, const void* V, int dt, int stride, const float* Z,
                                    const float* w0, const float* bonus, float* state, float* L, float* part,
                                    float* whole, const int32_t* cu, const int32_t* seq_slot, float* o, int n_seqs,
                                    int max_rows, int H, int d, void* stream) {
    if (n_seqs < 0 || n_seqs > 65535 || max_rows < 0 || max_rows > TM_SUB * 65535 || H <= 0 || H > 65535 || d <= 0 ||
        d > 128 || d % 4 || !illm_dtype_ok(dt) || stride < H * d || stride % 4 || !L || !part || !whole)
        return ILLM_ERR_ARG;
    if (n_seqs == 0 || max_rows == 0) return ILLM_OK;
    hipStream_t st = (hipStream_t)stream;
    hipLaunchKernelGGL(time_mix_decay_sums_kernel,
                       dim3((H * d + 255) / 256, (max_rows + TM_SUB - 1) / TM_SUB, n_seqs), dim3(256), 0, st, Z, w0, L,
                       cu, H * d);
    if (hipGetLastError() != hipSuccess) return ILLM_ERR_LAUNCH;
    if (dt == ILLM_BF16)
        return time_mix_chunks_launch<ILLM_BF16>(R, K, V, stride, L, bonus, state, part, whole, cu, seq_slot, o, n_seqs,
                                                 max_rows, H, d, st);
    return time_mix_chunks_launch<ILLM_F32>(R, K, V, stride, L, bonus, state, part, whole, cu, seq_slot, o, n_seqs,
                                            max_rows, H, d, st);
}
