// The delta rule with a removal vector over long steps, in chunks of RC tokens.  Per head, with the
// key size d, c_t = a_t u_t and D_t = diag(w_t):
//     S_t = D_t S_(t-1) - c_t (u_t^T S_(t-1)) + k_t v_t^T;   o_t = S_t^T r_t
// Within a chunk let P_t = D_1 .. D_t (a decay keeps at least exp(-rate) a token, so P and 1 / P of RC
// tokens stay well inside float32) and
//     u~_t = P_(t-1) u_t,  c~_t = c_t / P_t,  k~_t = k_t / P_t,  r~_t = P_t r_t.
// What the rule reads, y_t = S_(t-1)^T u_t, then solves (I + A) Y = U~ S_0 + B V with the strictly lower
// triangles A_tj = u~_t . c~_j, B_tj = u~_t . k~_j, and with the lower triangles M_tj = r~_t . k~_j,
// N_tj = r~_t . c~_j
//     O = R~ S_0 + M V - N Y,      S_end = P_RC (S_0 + K~^T V - C~^T Y).
//   removal_chunk_prepare  per (chunk, head), in parallel: the four triangles, W = (I + A)^-1 U~,
//                          Y0 = (I + A)^-1 B V (forward substitution, a thread a column), R' = R~ - N W,
//                          O0 = M V - N Y0
//   removal_chunk_carry    per (head, 16 value columns), chunk after chunk: Y = W S + Y0, O = R' S + O0,
//                          S <- P_RC (S + K~^T V - C~^T Y), S in the waves' accumulators
// All products on the matrix cores' float32 instructions (float32 operands, products and sums).  A row's
// sums run in another order than token by token: they differ in rounding only.
#include <math.h>

#include "api.h"
#include "common.h"

#define RC 32
typedef float rc_f32x16_t __attribute__((ext_vector_type(16)));
typedef float rc_f32x4_t __attribute__((ext_vector_type(4)));

// A chunk's pieces for one head, DP = 32 KT: W [RC][DP] | R' [RC][DP] | -C~^T [DP][RC] | K~^T [DP][RC] |
// V^T [DP][RC] | Y0^T [DP][RC] | O0^T [DP][RC] | P_RC [DP].  Chunk c of sequence b lies at place
// cu[b] / RC + b + c.
__host__ __device__ static inline size_t rc_floats(int DP) { return (size_t)DP * (7 * RC + 1); }

__device__ __forceinline__ float rc_sigmoid(float x) { return 1.0f / (1.0f + expf(-x)); }

// grid (chunks, H, sequences); 256 threads.
template <int DT, int KT>
__global__ void __launch_bounds__(256)
removal_chunk_prepare_kernel(const void* __restrict__ U, int u_stride, int r_off, int k_off, int v_off,
                             int a_off, const float* __restrict__ a_bias, const float* __restrict__ Z,
                             int z_stride, const float* __restrict__ w0, float rate, float* __restrict__ part,
                             const int32_t* __restrict__ cu, int H, int d) {
    constexpr int DP = 32 * KT, LD = DP + 1, GA = RC + 4, GL = RC + 1;
    __shared__ float ut[RC * LD], ct[RC * LD], kt[RC * LD], rt[RC * LD];
    __shared__ float vs[RC * DP], ys[RC * DP];
    __shared__ __attribute__((aligned(16))) float ga[RC * GA];
    __shared__ float gram[3][RC * GL];                  // B, M, N
    __shared__ float inv[RC];
    const int b = blockIdx.z, h = blockIdx.y, c = blockIdx.x, tid = threadIdx.x;
    const int r0 = cu[b], n = cu[b + 1] - r0, t0 = c * RC;
    if (t0 >= n) return;                                // the whole block
    const int nc = min(RC, n - t0);
    const int lane = tid & 63, w = wave_index(), col = lane & 31, half = lane >> 5;
    const size_t row0 = (size_t)(r0 + t0);
    float* dst = part + ((size_t)(r0 / RC + b + c) * H + h) * rc_floats(DP);
    float* const oW = dst;
    float* const oR = oW + RC * DP;
    float* const oC = oR + RC * DP;
    float* const oK = oC + RC * DP;
    float* const oV = oK + RC * DP;
    float* const oY = oV + RC * DP;
    float* const oO = oY + RC * DP;
    float* const oP = oO + RC * DP;

    for (int t = w; t < RC; t += 4) {
        float ss = 0.f;
        if (t < nc)
            for (int i = lane; i < d; i += 64) {
                const float k = ld_f(U, DT, (row0 + t) * u_stride + k_off + (size_t)h * d + i);
                ss = fmaf(k, k, ss);
            }
        ss = wave_sum(ss);
        if (lane == 0) inv[t] = 1.0f / sqrtf(ss + 1e-6f);
    }
    __syncthreads();
    {
        // a thread a channel and RC / NG tokens; the decays of the tokens before them are summed again
        constexpr int NG = 256 / DP, TG = RC / NG;
        const int ch = tid % DP, grp = tid / DP;
        if (grp < NG) {
            const bool in = ch < d;
            const int hc = h * d + (in ? ch : 0);
            const float bias0 = w0[hc], abias = a_bias[hc];
            auto log_decay = [&](int t) {
                return (in && t < nc) ? -rate * rc_sigmoid(Z[(row0 + t) * z_stride + hc] + bias0) : 0.f;
            };
            float L = 0.f;
#pragma unroll 4
            for (int t = 0; t < grp * TG; ++t) L += log_decay(t);
#pragma unroll 4
            for (int j = 0; j < TG; ++j) {
                const int t = grp * TG + j;
                float k = 0.f, r = 0.f, v = 0.f, a = 0.f;
                if (in && t < nc) {
                    const size_t at = (row0 + t) * u_stride + hc;
                    k = ld_f(U, DT, at + k_off);
                    r = ld_f(U, DT, at + r_off);
                    v = ld_f(U, DT, at + v_off);
                    a = rc_sigmoid(ld_f(U, DT, at + a_off) + abias);
                }
                const float before = expf(L);
                L += log_decay(t);
                const float P = expf(L), Q = expf(-L), u = k * inv[t];
                ut[t * LD + ch] = before * u;
                ct[t * LD + ch] = Q * (a * u);
                kt[t * LD + ch] = Q * k;
                rt[t * LD + ch] = P * r;
                vs[t * DP + ch] = v;
            }
            if (grp == NG - 1) oP[ch] = expf(L);
        }
    }
    __syncthreads();
    {
        const float* x = w < 2 ? ut : rt;
        const float* y = (w == 0 || w == 3) ? ct : kt;
        rc_f32x16_t g;
#pragma unroll
        for (int v = 0; v < 16; ++v) g[v] = 0.f;
#pragma unroll 8
        for (int s = 0; s < DP / 2; ++s)
            g = __builtin_amdgcn_mfma_f32_32x32x2f32(x[col * LD + 2 * s + half], y[col * LD + 2 * s + half], g, 0, 0, 0);
        float* to = w == 0 ? ga : gram[w - 1];
        const int ld = w == 0 ? GA : GL;
#pragma unroll
        for (int v = 0; v < 16; ++v) {
            const int t = 8 * (v >> 2) + 4 * half + (v & 3);
            to[t * ld + col] = (w < 2 ? col < t : col <= t) ? g[v] : 0.f;
        }
    }
    __syncthreads();
    if (w < KT) {                                       // B V
        rc_f32x16_t g;
#pragma unroll
        for (int v = 0; v < 16; ++v) g[v] = 0.f;
#pragma unroll
        for (int s = 0; s < RC / 2; ++s)
            g = __builtin_amdgcn_mfma_f32_32x32x2f32(gram[0][col * GL + 2 * s + half], vs[(2 * s + half) * DP + 32 * w + col],
                                                     g, 0, 0, 0);
#pragma unroll
        for (int v = 0; v < 16; ++v) ys[(8 * (v >> 2) + 4 * half + (v & 3)) * DP + 32 * w + col] = g[v];
    }
    __syncthreads();
    if (tid < 2 * DP) {                                 // (I + A) x = the column, row after row
        float* xs = tid < DP ? ut + tid : ys + (tid - DP);
        const int ld = tid < DP ? LD : DP;
        float x[RC];
#pragma unroll
        for (int t = 0; t < RC; ++t) {
            float s0 = xs[t * ld], s1 = 0.f;
#pragma unroll
            for (int j = 0; j < t; ++j) {
                if (j & 1) s1 = fmaf(-ga[t * GA + j], x[j], s1);
                else s0 = fmaf(-ga[t * GA + j], x[j], s0);
            }
            x[t] = s0 + s1;
        }
#pragma unroll
        for (int t = 0; t < RC; ++t) xs[t * ld] = x[t];
    }
    __syncthreads();
    if (w < KT) {
        const int n0 = 32 * w + col;
        rc_f32x16_t R, O;
#pragma unroll
        for (int v = 0; v < 16; ++v) {
            R[v] = rt[(8 * (v >> 2) + 4 * half + (v & 3)) * LD + n0];
            O[v] = 0.f;
        }
#pragma unroll
        for (int s = 0; s < RC / 2; ++s) {
            const int j = 2 * s + half;
            const float N = -gram[2][col * GL + j];
            R = __builtin_amdgcn_mfma_f32_32x32x2f32(N, ut[j * LD + n0], R, 0, 0, 0);
            O = __builtin_amdgcn_mfma_f32_32x32x2f32(N, ys[j * DP + n0], O, 0, 0, 0);
            O = __builtin_amdgcn_mfma_f32_32x32x2f32(gram[1][col * GL + j], vs[j * DP + n0], O, 0, 0, 0);
        }
#pragma unroll
        for (int v = 0; v < 16; ++v) oR[(8 * (v >> 2) + 4 * half + (v & 3)) * DP + n0] = R[v];
#pragma unroll
        for (int g = 0; g < 4; ++g)
            *(float4*)(oO + (size_t)n0 * RC + 8 * g + 4 * half) = make_float4(O[4 * g], O[4 * g + 1], O[4 * g + 2], O[4 * g + 3]);
    }
    for (int e = tid; e < RC * DP; e += 256) oW[e] = ut[(e / DP) * LD + e % DP];
    for (int e = tid; e < (RC / 4) * DP; e += 256) {
        const int ch = e % DP, t = 4 * (e / DP);
        *(float4*)(oC + ch * RC + t) = make_float4(-ct[t * LD + ch], -ct[(t + 1) * LD + ch], -ct[(t + 2) * LD + ch], -ct[(t + 3) * LD + ch]);
        *(float4*)(oK + ch * RC + t) = make_float4(kt[t * LD + ch], kt[(t + 1) * LD + ch], kt[(t + 2) * LD + ch], kt[(t + 3) * LD + ch]);
        *(float4*)(oV + ch * RC + t) = make_float4(vs[t * DP + ch], vs[(t + 1) * DP + ch], vs[(t + 2) * DP + ch], vs[(t + 3) * DP + ch]);
        *(float4*)(oY + ch * RC + t) = make_float4(ys[t * DP + ch], ys[(t + 1) * DP + ch], ys[(t + 2) * DP + ch], ys[(t + 3) * DP + ch]);
    }
}

// What a wave reads of a chunk: with lane = m + 16 q, W and R' rows 16 tt + m at its own key rows 32 w + 16
// a + 4 q .. + 3, -C~^T and K~^T rows 32 w + 16 a + m at tokens 16 tt + 4 q .. + 3, and V^T, Y0^T of the
// block's value column m at those tokens.
struct RcPiece {
    float4 W[2][2], R[2][2], C[2][2], K[2][2], V[2], Y[2], O, P[2];
};

// grid (H, ceil(d / 16), sequences) (a head's blocks lie 8 or more apart in number, so on one die when H is
// a multiple of 8, and share its cache); 256 threads: wave w holds rows [32 w, 32 w + 32) of the block's
// 16 columns of S, two tiles of 16 x 16.  MFMA 16x16x4: in step i a lane's quarter q stands for row 4 q + i
// of a tile, in both operands, so that an accumulator is the next product's second operand as it stands.
template <int KT>
__global__ void __launch_bounds__(256, 1)
removal_chunk_carry_kernel(const float* __restrict__ part, float* __restrict__ state,
                           const int32_t* __restrict__ cu, const int32_t* __restrict__ seq_slot,
                           float* __restrict__ o, int H, int d) {
    constexpr int DP = 32 * KT;
    __shared__ float4 red[2][KT][4][64];
    const int h = blockIdx.x, n0 = blockIdx.y * 16, b = blockIdx.z;
    const int r0 = cu[b], n = cu[b + 1] - r0;
    if (n <= 0) return;                                 // the whole block
    const int lane = threadIdx.x & 63, w = wave_index(), m = lane & 15, q = lane >> 4;
    const bool works = w < KT;
    const int chunks = (n + RC - 1) / RC;
    const size_t step = (size_t)H * rc_floats(DP);
    const float* base = part + ((size_t)(r0 / RC + b) * H + h) * rc_floats(DP);
    float* sp = state + (((size_t)seq_slot[b] * H + h) * d) * d + n0 + m;
    const bool col_in = n0 + m < d;
    rc_f32x4_t s[2];
#pragma unroll
    for (int a = 0; a < 2; ++a)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int row = 32 * w + 16 * a + 4 * q + i;
            s[a][i] = (works && col_in && row < d) ? sp[(size_t)row * d] : 0.f;
        }
    const int wr = works ? w : 0;                       // (a wave without rows reads wave 0's pieces)
    auto fetch = [&](int c, RcPiece& x) __attribute__((always_inline)) {
        const float* p = base + (size_t)c * step;
#pragma unroll
        for (int tt = 0; tt < 2; ++tt) {
#pragma unroll
            for (int a = 0; a < 2; ++a) {
                const int row = 32 * wr + 16 * a;
                x.W[tt][a] = *(const float4*)(p + (16 * tt + m) * DP + row + 4 * q);
                x.R[tt][a] = *(const float4*)(p + (RC + 16 * tt + m) * DP + row + 4 * q);
                x.C[tt][a] = *(const float4*)(p + 2 * RC * DP + (row + m) * RC + 16 * tt + 4 * q);
                x.K[tt][a] = *(const float4*)(p + 3 * RC * DP + (row + m) * RC + 16 * tt + 4 * q);
            }
            x.V[tt] = *(const float4*)(p + 4 * RC * DP + (n0 + m) * RC + 16 * tt + 4 * q);
            x.Y[tt] = *(const float4*)(p + 5 * RC * DP + (n0 + m) * RC + 16 * tt + 4 * q);
        }
        x.O = *(const float4*)(p + 6 * RC * DP + (n0 + m) * RC + 16 * (w & 1) + 4 * q);
#pragma unroll
        for (int a = 0; a < 2; ++a) x.P[a] = *(const float4*)(p + 7 * RC * DP + 32 * wr + 16 * a + 4 * q);
    };
#define F4(X_, I_) (((const float*)&(X_))[I_])
    RcPiece x, nx;
    fetch(0, x);
    for (int c = 0; c < chunks; ++c) {
        fetch(c + 1 < chunks ? c + 1 : c, nx);          // (the last chunk is asked for twice)
        const int buf = c & 1;
        if (works) {
            rc_f32x4_t z[4];
#pragma unroll
            for (int t = 0; t < 4; ++t) z[t] = (rc_f32x4_t){0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int a = 0; a < 2; ++a)
#pragma unroll
                for (int i = 0; i < 4; ++i)
#pragma unroll
                    for (int tt = 0; tt < 2; ++tt) {
                        z[tt] = __builtin_amdgcn_mfma_f32_16x16x4f32(F4(x.W[tt][a], i), s[a][i], z[tt], 0, 0, 0);
                        z[2 + tt] = __builtin_amdgcn_mfma_f32_16x16x4f32(F4(x.R[tt][a], i), s[a][i], z[2 + tt], 0, 0, 0);
                    }
#pragma unroll
            for (int t = 0; t < 4; ++t) red[buf][w][t][lane] = make_float4(z[t][0], z[t][1], z[t][2], z[t][3]);
#pragma unroll
            for (int tt = 0; tt < 2; ++tt)
#pragma unroll
                for (int i = 0; i < 4; ++i)
#pragma unroll
                    for (int a = 0; a < 2; ++a)
                        s[a] = __builtin_amdgcn_mfma_f32_16x16x4f32(F4(x.K[tt][a], i), F4(x.V[tt], i), s[a], 0, 0, 0);
        }
        __syncthreads();
        // (two buffers in turn: nobody writes this one again before everybody has passed the next barrier)
        if (works) {
#pragma unroll
            for (int tt = 0; tt < 2; ++tt) {
                float4 y = x.Y[tt];
#pragma unroll
                for (int k = 0; k < KT; ++k) {
                    const float4 z = red[buf][k][tt][lane];
                    y.x += z.x; y.y += z.y; y.z += z.z; y.w += z.w;
                }
#pragma unroll
                for (int i = 0; i < 4; ++i)
#pragma unroll
                    for (int a = 0; a < 2; ++a)
                        s[a] = __builtin_amdgcn_mfma_f32_16x16x4f32(F4(x.C[tt][a], i), F4(y, i), s[a], 0, 0, 0);
            }
#pragma unroll
            for (int a = 0; a < 2; ++a)
#pragma unroll
                for (int i = 0; i < 4; ++i) s[a][i] *= F4(x.P[a], i);
        }
        if (w < 2) {                                    // tokens 16 w .. 16 w + 15 of the chunk
            float4 y = x.O;
#pragma unroll
            for (int k = 0; k < KT; ++k) {
                const float4 z = red[buf][k][2 + w][lane];
                y.x += z.x; y.y += z.y; y.z += z.z; y.w += z.w;
            }
            if (col_in) {
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    const int t = c * RC + 16 * w + 4 * q + i;
                    if (t < n) o[((size_t)(r0 + t) * H + h) * d + n0 + m] = F4(y, i);
                }
            }
        }
        x = nx;
    }
#undef F4
#pragma unroll
    for (int a = 0; a < 2; ++a)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int row = 32 * w + 16 * a + 4 * q + i;
            if (works && col_in && row < d) sp[(size_t)row * d] = s[a][i];
        }
}

extern "C" int illm_removal_chunk(void) { return RC; }
extern "C" int illm_removal_chunk_floats(int d) { return d > 0 && d <= 128 ? (int)rc_floats((d + 31) / 32 * 32) : 0; }

extern "C" int illm_removal_chunks(const void* U, int dt, int u_stride, int r_off, int k_off, int v_off, int a_off,
                                   const float* a_bias, const float* Z, int z_stride, const float* w0, float rate,
                                   float* state, float* part, const int32_t* cu, const int32_t* seq_slot, float* o,
                                   int n_seqs, int max_rows, int H, int d, void* stream) {
    auto cols = [&](int off) { return off >= 0 && off + H * d <= u_stride; };
    // (1 / P of a chunk must stay inside float32: 32 rate well below 88)
    if (n_seqs < 0 || n_seqs > 65535 || max_rows < 0 || H <= 0 || H > 65535 || d <= 0 || d > 128 || !illm_dtype_ok(dt) ||
        !cols(r_off) || !cols(k_off) || !cols(v_off) || !cols(a_off) || z_stride < H * d || !part ||
        !(rate >= 0.f && rate <= 1.25f))
        return ILLM_ERR_ARG;
    if (n_seqs == 0 || max_rows == 0) return ILLM_OK;
    hipStream_t st = (hipStream_t)stream;
    const dim3 grid((max_rows + RC - 1) / RC, H, n_seqs), grid2(H, (d + 15) / 16, n_seqs);
#define GO_D(DT_, KT_)                                                                                         \
    hipLaunchKernelGGL((removal_chunk_prepare_kernel<DT_, KT_>), grid, dim3(256), 0, st, U, u_stride, r_off, k_off, \
                       v_off, a_off, a_bias, Z, z_stride, w0, rate, part, cu, H, d)
#define GO(KT_)                                                                                                \
    do {                                                                                                       \
        if (dt == ILLM_BF16) GO_D(ILLM_BF16, KT_); else GO_D(ILLM_F32, KT_);                                   \
        if (hipGetLastError() != hipSuccess) return ILLM_ERR_LAUNCH;                                           \
        hipLaunchKernelGGL(removal_chunk_carry_kernel<KT_>, grid2, dim3(256), 0, st, part, state, cu, seq_slot, o, H, d); \
    } while (0)
    switch ((d + 31) / 32) {
        case 1: GO(1); break;
        case 2: GO(2); break;
        case 3: GO(3); break;
        default: GO(4); break;
    }
#undef GO
#undef GO_D
    return illm_launch_status();
}
