// Row-wise kernels: embedding rows, residual add + RMS norm, SiLU-multiply,
// rotation of q/k with the store of k/v into the paged cache.
//
// Formulas as the reference computes them: embedding row copy
// (src/kern/naive/naive.cpp:43-54), RMS norm = x * 1/sqrt(mean(x^2) + eps), then
// the weight (naive.cpp:186-207, src/core/op.cpp:37-47), silu(x) = x / (1 + exp(-x))
// (naive.cpp:80-89), rotation of pairs (i, i + hd/2) by pos * base^(-2i/rot)
// (naive.cpp:389-414) or of pairs (2i, 2i+1) (naive.cpp:415-440).  The reference
// runs each as a kernel of its own (src/kern/gpu/kernel_gpu.cu:127-148, :260-294,
// :183-258, :343-401); here the residual add is fused with the norm and the cache
// store with the rotation.
#include "api.h"
#include "common.h"

// ---------------------------------------------------------------- embedding
__global__ void embed_kernel(const int32_t* __restrict__ tokens, const void* __restrict__ table,
                             int table_dt, float* __restrict__ out, int E, int V, float scale) {
    const int t = blockIdx.x;
    int id = tokens[t];
    id = id < 0 ? 0 : (id >= V ? V - 1 : id);
    const size_t src = (size_t)id * E, dst = (size_t)t * E;
    for (int i = threadIdx.x; i < E; i += blockDim.x)
        out[dst + i] = ld_f(table, table_dt, src + i) * scale;
}

extern "C" int illm_embed_scaled(const int32_t* tokens, const void* table, int table_dt, float* out,
                                 int T, int E, int V, float scale, void* stream) {
    if (T < 0 || E <= 0 || V <= 0 || !illm_dtype_ok(table_dt)) return ILLM_ERR_ARG;
    if (T == 0) return ILLM_OK;
    hipLaunchKernelGGL(embed_kernel, dim3(T), dim3(256), 0, (hipStream_t)stream, tokens, table,
                       table_dt, out, E, V, scale);
    return illm_launch_status();
}

extern "C" int illm_embed(const int32_t* tokens, const void* table, int table_dt, float* out,
                          int T, int E, int V, void* stream) {
    return illm_embed_scaled(tokens, table, table_dt, out, T, E, V, 1.0f, stream);
}

// The token's row under an RMS norm: out = v / sqrt(mean(v^2) + eps) * w with v = table[id] * scale.  `copy`
// (null: none) takes the rows a second time.  grid (rows); 256 threads, NV groups of 4 columns a thread, the row
// and the weights asked for together; NV 0: any width.
template <int NV>
__global__ void __launch_bounds__(256)
embed_norm_kernel(const int32_t* __restrict__ tokens, const void* __restrict__ table, int table_dt,
                  const void* __restrict__ w, int w_dt, float* __restrict__ out, float* __restrict__ copy, int E,
                  int V, float scale, float eps) {
    __shared__ float red[16];
    const int t = blockIdx.x;
    int id = tokens[t];
    id = id < 0 ? 0 : (id >= V ? V - 1 : id);
    if (NV > 0) {
        const size_t n4 = E / 4, src = (size_t)id * n4, dst = (size_t)t * n4;
        float4 v[NV ? NV : 1], g[NV ? NV : 1];
        float ss = 0.f;
#pragma unroll
        for (int k = 0; k < NV; ++k) {
            const size_t i = threadIdx.x + 256 * k;
            v[k] = i < n4 ? ld_f4(table, table_dt, src + i) : make_float4(0.f, 0.f, 0.f, 0.f);
            g[k] = i < n4 ? ld_f4(w, w_dt, i) : make_float4(0.f, 0.f, 0.f, 0.f);
        }
#pragma unroll
        for (int k = 0; k < NV; ++k) {
            v[k].x *= scale; v[k].y *= scale; v[k].z *= scale; v[k].w *= scale;
            ss += (v[k].x * v[k].x + v[k].y * v[k].y) + (v[k].z * v[k].z + v[k].w * v[k].w);
        }
        ss = block_sum(ss, red);
        const float inv = 1.0f / sqrtf(ss / (float)E + eps);
#pragma unroll
        for (int k = 0; k < NV; ++k) {
            const size_t i = threadIdx.x + 256 * k;
            if (i >= n4) continue;
            const float4 y = make_float4(v[k].x * inv * g[k].x, v[k].y * inv * g[k].y, v[k].z * inv * g[k].z,
                                         v[k].w * inv * g[k].w);
            ((float4*)out)[dst + i] = y;
            if (copy) ((float4*)copy)[dst + i] = y;
        }
        return;
    }
    const size_t src = (size_t)id * E, dst = (size_t)t * E;
    float ss = 0.f;
    for (int i = threadIdx.x; i < E; i += 256) {
        const float v = ld_f(table, table_dt, src + i) * scale;
        ss = fmaf(v, v, ss);
    }
    ss = block_sum(ss, red);
    const float inv = 1.0f / sqrtf(ss / (float)E + eps);
    for (int i = threadIdx.x; i < E; i += 256) {
        const float y = (ld_f(table, table_dt, src + i) * scale * inv) * ld_f(w, w_dt, i);
        out[dst + i] = y;
        if (copy) copy[dst + i] = y;
    }
}

extern "C" int illm_embed_norm(const int32_t* tokens, const void* table, int table_dt, const void* w, int w_dt,
                               float* out, float* copy, int T, int E, int V, float scale, float eps, void* stream) {
    if (T < 0 || E <= 0 || V <= 0 || !illm_dtype_ok(table_dt) || !illm_dtype_ok(w_dt)) return ILLM_ERR_ARG;
    if (T == 0) return ILLM_OK;
#define GO(NV_)                                                                                            \
    hipLaunchKernelGGL(embed_norm_kernel<NV_>, dim3(T), dim3(256), 0, (hipStream_t)stream, tokens, table, table_dt, w, \
                       w_dt, out, copy, E, V, scale, eps)
    if (E % 4 || E > 8192) GO(0);
    else if (E <= 1024) GO(1);
    else if (E <= 2048) GO(2);
    else if (E <= 4096) GO(4);
    else GO(8);
#undef GO
    return illm_launch_status();
}

// A copy of float32 rows (a kernel and no memory-copy command, for code under graph capture).
__global__ void __launch_bounds__(256)
copy_rows_kernel(const float* __restrict__ x, float* __restrict__ out, size_t n) {
    const size_t step = (size_t)gridDim.x * 256;
    for (size_t i = (size_t)blockIdx.x * 256 + threadIdx.x; i < n; i += step) out[i] = x[i];
}

extern "C" int illm_copy_rows(const float* x, float* out, size_t n, void* stream) {
    if (!x || !out) return ILLM_ERR_ARG;
    if (n == 0) return ILLM_OK;
    const size_t blocks = (n + 255) / 256;
    hipLaunchKernelGGL(copy_rows_kernel, dim3(blocks < 4096 ? blocks : 4096), dim3(256), 0, (hipStream_t)stream, x, out, n);
    return illm_launch_status();
}

// Token row times a scale, plus a row of a table hashed by the pair (previous token, token), plus a
// learned row of the position:
//     out = table[id] * scale + pairs[(prev * mul_prev + id * mul_cur) mod buckets] + places[pos]
// A sequence's first token (position 0) takes row `buckets` of `pairs`, its last.  The token before a
// row is the row above it if that belongs to the same slot, else `last_token[slot]`: what the
// sequence's last step left.  `pairs` or `places` may be null (that addend is left out).
// `remember`: every sequence brings one row, and the row's thread also leaves its token in
// `last_token`; steps of several rows a sequence call illm_remember_last afterwards.
__global__ void embed_pairs_kernel(const int32_t* __restrict__ tokens, const int32_t* __restrict__ row_pos,
                                   const int32_t* __restrict__ row_slot, const void* __restrict__ table,
                                   int table_dt, const void* __restrict__ pairs, int pairs_dt,
                                   const void* __restrict__ places, int places_dt,
                                   int32_t* __restrict__ last_token, float* __restrict__ out, int E, int V,
                                   int buckets, int mul_prev, int mul_cur, int n_places, float scale,
                                   int remember) {
    const int t = blockIdx.x;
    int id = tokens[t];
    id = id < 0 ? 0 : (id >= V ? V - 1 : id);
    int pos = row_pos[t];
    pos = pos < 0 ? 0 : (pos >= n_places ? n_places - 1 : pos);
    const int slot = row_slot[t];
    int pair = buckets;
    if (pairs && row_pos[t] > 0) {
        int prev = (t > 0 && row_slot[t - 1] == slot) ? tokens[t - 1] : last_token[slot];
        prev = prev < 0 ? 0 : (prev >= V ? V - 1 : prev);
        pair = (int)(((long long)prev * mul_prev + (long long)id * mul_cur) % buckets);
    }
    const size_t src = (size_t)id * E, dst = (size_t)t * E;
    for (int i = threadIdx.x; i < E; i += blockDim.x) {
        float v = ld_f(table, table_dt, src + i) * scale;
        if (pairs) v += ld_f(pairs, pairs_dt, (size_t)pair * E + i);
        if (places) v += ld_f(places, places_dt, (size_t)pos * E + i);
        out[dst + i] = v;
    }
    if (remember && last_token && threadIdx.x == 0) last_token[slot] = id;
}

extern "C" int illm_embed_pairs(const int32_t* tokens, const int32_t* row_pos, const int32_t* row_slot,
                                const void* table, int table_dt, const void* pairs, int pairs_dt,
                                const void* places, int places_dt, int32_t* last_token, float* out,
                                int T, int E, int V, int buckets, int mul_prev, int mul_cur,
                                int n_places, float scale, int remember, void* stream) {
    if (T < 0 || E <= 0 || V <= 0 || !illm_dtype_ok(table_dt) || (pairs && (!illm_dtype_ok(pairs_dt) ||
        buckets <= 0 || mul_prev < 0 || mul_cur < 0 || !last_token)) || (places && (!illm_dtype_ok(places_dt) ||
        n_places <= 0)))
        return ILLM_ERR_ARG;
    if (T == 0) return ILLM_OK;
    hipLaunchKernelGGL(embed_pairs_kernel, dim3(T), dim3(256), 0, (hipStream_t)stream, tokens, row_pos,
                       row_slot, table, table_dt, pairs, pairs_dt, places, places_dt, last_token, out, E, V,
                       buckets, mul_prev, mul_cur, places ? n_places : 1, scale, remember);
    return illm_launch_status();
}

// last_token[seq_slot[b]] = the last token of sequence b's rows in this step (none: left as it is).
__global__ void remember_last_kernel(const int32_t* __restrict__ tokens, const int32_t* __restrict__ cu,
                                     const int32_t* __restrict__ seq_slot, int32_t* __restrict__ last_token,
                                     int n_seqs) {
    const int b = blockIdx.x * blockDim.x + threadIdx.x;
    if (b >= n_seqs) return;
    const int end = cu[b + 1];
    if (end > cu[b]) last_token[seq_slot[b]] = tokens[end - 1];
}

extern "C" int illm_remember_last(const int32_t* tokens, const int32_t* cu, const int32_t* seq_slot,
                                  int32_t* last_token, int n_seqs, void* stream) {
    if (n_seqs < 0) return ILLM_ERR_ARG;
    if (n_seqs == 0) return ILLM_OK;
    hipLaunchKernelGGL(remember_last_kernel, dim3((n_seqs + 63) / 64), dim3(64), 0, (hipStream_t)stream,
                       tokens, cu, seq_slot, last_token, n_seqs);
    return illm_launch_status();
}

// ---------------------------------------------------------------- sums and activations by element
__global__ void sum_rows_kernel(const void* __restrict__ a, int a_dt, const void* __restrict__ b,
                                int b_dt, float* __restrict__ out, size_t n) {
    const size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
    if (i < n) out[i] = ld_f(a, a_dt, i) + ld_f(b, b_dt, i);
}

extern "C" int illm_sum_rows(const void* a, int a_dt, const void* b, int b_dt, float* out,
                             size_t n, void* stream) {
    if (!illm_dtype_ok(a_dt) || !illm_dtype_ok(b_dt)) return ILLM_ERR_ARG;
    if (n == 0) return ILLM_OK;
    hipLaunchKernelGGL(sum_rows_kernel, dim3((unsigned)((n + 255) / 256)), dim3(256), 0,
                       (hipStream_t)stream, a, a_dt, b, b_dt, out, n);
    return illm_launch_status();
}

__global__ void sum_rows_scaled_kernel(const void* __restrict__ a, int a_dt, float sa,
                                       const void* __restrict__ b, int b_dt, float sb,
                                       float* __restrict__ out, size_t n) {
    const size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
    if (i < n) out[i] = sa * ld_f(a, a_dt, i) + sb * ld_f(b, b_dt, i);
}

extern "C" int illm_sum_rows_scaled(const void* a, int a_dt, float sa, const void* b, int b_dt,
                                    float sb, float* out, size_t n, void* stream) {
    if (!illm_dtype_ok(a_dt) || !illm_dtype_ok(b_dt)) return ILLM_ERR_ARG;
    if (n == 0) return ILLM_OK;
    hipLaunchKernelGGL(sum_rows_scaled_kernel, dim3((unsigned)((n + 255) / 256)), dim3(256), 0,
                       (hipStream_t)stream, a, a_dt, sa, b, b_dt, sb, out, n);
    return illm_launch_status();
}

__global__ void relu_squared_kernel(const void* __restrict__ x, void* __restrict__ out, int dt,
                                    size_t n) {
    const size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
    if (i >= n) return;
    const float v = fmaxf(ld_f(x, dt, i), 0.f);
    st_f(out, dt, i, v * v);
}

// 0.5 z (1 + tanh(sqrt(2 / pi) (z + 0.044715 z^3))), the tanh form of GELU.
__global__ void gelu_tanh_kernel(const void* __restrict__ x, void* __restrict__ out, int dt, size_t n) {
    const size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
    if (i >= n) return;
    const float z = ld_f(x, dt, i);
    st_f(out, dt, i, 0.5f * z * (1.0f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z))));
}

__device__ __forceinline__ float gelu_tanh_f(float z) {
    return 0.5f * z * (1.0f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
}

// bfloat16 with n % 8 == 0: 8 values (16 bytes) a thread
__global__ void __launch_bounds__(256)
gelu_tanh_bf16x8_kernel(const bf16_t* __restrict__ x, bf16_t* __restrict__ out, size_t n8) {
    const size_t i = (size_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= n8) return;
    const uint4 v = ((const uint4*)x)[i];
    const uint32_t w[4] = {v.x, v.y, v.z, v.w};
    uint32_t o[4];
#pragma unroll
    for (int k = 0; k < 4; ++k)
        o[k] = pack_bf16x2(gelu_tanh_f(__uint_as_float(w[k] << 16)), gelu_tanh_f(__uint_as_float(w[k] & 0xffff0000u)));
    ((uint4*)out)[i] = make_uint4(o[0], o[1], o[2], o[3]);
}

extern "C" int illm_gelu_tanh(const void* x, void* out, int dt, size_t n, void* stream) {
    if (!illm_dtype_ok(dt)) return ILLM_ERR_ARG;
    if (n == 0) return ILLM_OK;
    if (dt == ILLM_BF16 && n % 8 == 0 && n / 8 / 256 < 0x7fffffffu) {
        hipLaunchKernelGGL(gelu_tanh_bf16x8_kernel, dim3((unsigned)((n / 8 + 255) / 256)), dim3(256), 0,
                           (hipStream_t)stream, (const bf16_t*)x, (bf16_t*)out, n / 8);
        return illm_launch_status();
    }
    hipLaunchKernelGGL(gelu_tanh_kernel, dim3((unsigned)((n + 255) / 256)), dim3(256), 0,
                       (hipStream_t)stream, x, out, dt, n);
    return illm_launch_status();
}

// xIELU with two numbers on the device, par = (cp, cn): z > 0: cp z^2 + z / 2; z <= 0: cn (e^z - 1 - z) + z / 2.
__device__ __forceinline__ float xielu_f(float z, float cp, float cn) {
    return (z > 0.f ? cp * z * z : cn * (expm1f(z) - z)) + 0.5f * z;
}

__global__ void xielu_kernel(const void* __restrict__ x, const float* __restrict__ par, void* __restrict__ out,
                             int dt, size_t n) {
    const size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
    if (i < n) st_f(out, dt, i, xielu_f(ld_f(x, dt, i), par[0], par[1]));
}

// bfloat16 with n % 8 == 0: 8 values (16 bytes) a thread; ACT 0: max(z, 0)^2, 1: xIELU
template <int ACT>
__global__ void __launch_bounds__(256)
act_bf16x8_kernel(const bf16_t* __restrict__ x, const float* __restrict__ par, bf16_t* __restrict__ out, size_t n8) {
    const size_t i = (size_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= n8) return;
    const float cp = ACT ? par[0] : 0.f, cn = ACT ? par[1] : 0.f;
    auto act = [&](float z) {
        if (ACT) return xielu_f(z, cp, cn);
        z = fmaxf(z, 0.f);
        return z * z;
    };
    const uint4 v = ((const uint4*)x)[i];
    const uint32_t w[4] = {v.x, v.y, v.z, v.w};
    uint32_t o[4];
#pragma unroll
    for (int k = 0; k < 4; ++k)
        o[k] = pack_bf16x2(act(__uint_as_float(w[k] << 16)), act(__uint_as_float(w[k] & 0xffff0000u)));
    ((uint4*)out)[i] = make_uint4(o[0], o[1], o[2], o[3]);
}

extern "C" int illm_xielu(const void* x, const float* par, void* out, int dt, size_t n, void* stream) {
    if (!illm_dtype_ok(dt) || !par) return ILLM_ERR_ARG;
    if (n == 0) return ILLM_OK;
    if (dt == ILLM_BF16 && n % 8 == 0 && n / 8 / 256 < 0x7fffffffu) {
        hipLaunchKernelGGL(act_bf16x8_kernel<1>, dim3((unsigned)((n / 8 + 255) / 256)), dim3(256), 0,
                           (hipStream_t)stream, (const bf16_t*)x, par, (bf16_t*)out, n / 8);
        return illm_launch_status();
    }
    hipLaunchKernelGGL(xielu_kernel, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, (hipStream_t)stream, x,
                       par, out, dt, n);
    return illm_launch_status();
}

extern "C" int illm_relu_squared(const void* x, void* out, int dt, size_t n, void* stream) {
    if (!illm_dtype_ok(dt)) return ILLM_ERR_ARG;
    if (n == 0) return ILLM_OK;
    if (dt == ILLM_BF16 && n % 8 == 0 && n / 8 / 256 < 0x7fffffffu) {
        hipLaunchKernelGGL(act_bf16x8_kernel<0>, dim3((unsigned)((n / 8 + 255) / 256)), dim3(256), 0,
                           (hipStream_t)stream, (const bf16_t*)x, (const float*)nullptr, (bf16_t*)out, n / 8);
        return illm_launch_status();
    }
    hipLaunchKernelGGL(relu_squared_kernel, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, (hipStream_t)stream,
                       x, out, dt, n);
    return illm_launch_status();
}

// ---------------------------------------------------------------- add + rmsnorm
// One block per row.  The sum of squares is taken in float32 in an order that
// depends on E and the block size only, never on the row's place in the batch.
// `delta` may be `planes` arrays of the same shape, `plane_stride` elements apart (the sums of
// a product whose K was split): they are added in order.
__device__ __forceinline__ float ld_planes(const void* delta, int dt, size_t i, int planes,
                                           size_t plane_stride) {
    float d = ld_f(delta, dt, i);
    for (int s = 1; s < planes; ++s) d += ld_f(delta, dt, i + s * plane_stride);
    return d;
}

__global__ void add_rmsnorm_kernel(float* __restrict__ x, const void* __restrict__ delta,
                                   int delta_dt, int planes, size_t plane_stride,
                                   const void* __restrict__ delta2, int delta2_dt,
                                   const void* __restrict__ w, int w_dt,
                                   void* __restrict__ out, int out_dt,
                                   const int32_t* __restrict__ row_idx, int E, float eps,
                                   const void* __restrict__ w2, void* __restrict__ out2) {
    __shared__ float red[16];
    const int r = blockIdx.x;
    const int in_row = row_idx ? row_idx[r] : r;
    const size_t ib = (size_t)in_row * E, ob = (size_t)r * E;
    float ss = 0.f;
    for (int i = threadIdx.x; i < E; i += blockDim.x) {
        float v = x[ib + i];
        if (delta) {
            float d = ld_planes(delta, delta_dt, ib + i, planes, plane_stride);
            if (delta2) d += ld_f(delta2, delta2_dt, ib + i);
            v += d;
            if (!row_idx) x[ib + i] = v;
        }
        ss += v * v;
    }
    ss = block_sum(ss, red);
    const float scale = 1.0f / sqrtf(ss / (float)E + eps);
    for (int i = threadIdx.x; i < E; i += blockDim.x) {
        float v = x[ib + i];
        if (delta && row_idx) {
            float d = ld_planes(delta, delta_dt, ib + i, planes, plane_stride);
            if (delta2) d += ld_f(delta2, delta2_dt, ib + i);
            v += d;
        }
        st_f(out, out_dt, ob + i, (v * scale) * ld_f(w, w_dt, i));
        if (out2) st_f(out2, out_dt, ob + i, (v * scale) * ld_f(w2, w_dt, i));
    }
}

// The same with every element of the row held in registers: each thread owns NV
// groups of 4 consecutive floats, all loads are issued before the first use, and x is
// read once.  Needs E % 4 == 0 and E <= 1024 * NV.
__device__ __forceinline__ float4 ld4_f(const void* p, int dt, size_t i4) {
    if (dt == ILLM_BF16) {
        const uint2 u = ((const uint2*)p)[i4];
        return make_float4(__uint_as_float(u.x << 16), __uint_as_float(u.x & 0xffff0000u),
                           __uint_as_float(u.y << 16), __uint_as_float(u.y & 0xffff0000u));
    }
    return ((const float4*)p)[i4];
}

__device__ __forceinline__ void st4_f(void* p, int dt, size_t i4, float4 v) {
    if (dt == ILLM_BF16) {
        uint2 u;
        u.x = pack_bf16x2(v.x, v.y);
        u.y = pack_bf16x2(v.z, v.w);
        ((uint2*)p)[i4] = u;
    } else {
        ((float4*)p)[i4] = v;
    }
}

template <int NV, int TH>
__global__ void __launch_bounds__(TH)
add_rmsnorm_vec_kernel(float* __restrict__ x, const void* __restrict__ delta, int delta_dt,
                       int planes, size_t plane_stride4, const void* __restrict__ delta2,
                       int delta2_dt,
                       const void* __restrict__ w, int w_dt, void* __restrict__ out, int out_dt,
                       const int32_t* __restrict__ row_idx, int E, float eps,
                       const void* __restrict__ w2, void* __restrict__ out2) {
    __shared__ float red[16];
    const int r = blockIdx.x;
    const int in_row = row_idx ? row_idx[r] : r;
    const int E4 = E >> 2;
    const size_t ib = (size_t)in_row * E4, ob = (size_t)r * E4;
    float4 v[NV], wv[NV];
#pragma unroll
    for (int j = 0; j < NV; ++j) {
        const int i = threadIdx.x + TH * j;
        v[j] = make_float4(0.f, 0.f, 0.f, 0.f);
        wv[j] = v[j];
        if (i < E4) {
            v[j] = ((const float4*)x)[ib + i];
            wv[j] = ld4_f(w, w_dt, i);
        }
    }
    if (delta) {
#pragma unroll
        for (int j = 0; j < NV; ++j) {
            const int i = threadIdx.x + TH * j;
            if (i < E4) {
                float4 d = ld4_f(delta, delta_dt, ib + i);
                // the planes of a split product, four loads at a time, added in order
                for (int s0 = 1; s0 < planes; s0 += 4) {
                    float4 e[4];
#pragma unroll
                    for (int t = 0; t < 4; ++t)
                        e[t] = s0 + t < planes
                                   ? ld4_f(delta, delta_dt, ib + i + (size_t)(s0 + t) * plane_stride4)
                                   : make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
                    for (int t = 0; t < 4; ++t) {
                        d.x += e[t].x; d.y += e[t].y; d.z += e[t].z; d.w += e[t].w;
                    }
                }
                if (delta2) {                         // a second addend: (delta + delta2) first
                    const float4 e2 = ld4_f(delta2, delta2_dt, ib + i);
                    d.x += e2.x; d.y += e2.y; d.z += e2.z; d.w += e2.w;
                }
                v[j].x += d.x; v[j].y += d.y; v[j].z += d.z; v[j].w += d.w;
                if (!row_idx) ((float4*)x)[ib + i] = v[j];
            }
        }
    }
    float ss = 0.f;
#pragma unroll
    for (int j = 0; j < NV; ++j)
        ss += v[j].x * v[j].x + v[j].y * v[j].y + v[j].z * v[j].z + v[j].w * v[j].w;
    ss = block_sum(ss, red);
    const float scale = 1.0f / sqrtf(ss / (float)E + eps);
#pragma unroll
    for (int j = 0; j < NV; ++j) {
        const int i = threadIdx.x + TH * j;
        if (i < E4) {
            st4_f(out, out_dt, ob + i,
                  make_float4((v[j].x * scale) * wv[j].x, (v[j].y * scale) * wv[j].y,
                              (v[j].z * scale) * wv[j].z, (v[j].w * scale) * wv[j].w));
            if (out2) {                               // the same rows under a second norm's weight
                const float4 w2v = ld4_f(w2, w_dt, i);
                st4_f(out2, out_dt, ob + i,
                      make_float4((v[j].x * scale) * w2v.x, (v[j].y * scale) * w2v.y,
                                  (v[j].z * scale) * w2v.z, (v[j].w * scale) * w2v.w));
            }
        }
    }
}

extern "C" int illm_add2_rmsnorm_two(float* x, const void* delta, int delta_dt, int planes,
                                     size_t plane_stride, const void* delta2, int delta2_dt,
                                     const void* w, const void* w2, int w_dt, void* out, void* out2,
                                     int out_dt, const int32_t* row_idx, int rows, int E, float eps,
                                     void* stream) {
    if ((w2 == nullptr) != (out2 == nullptr)) return ILLM_ERR_ARG;
    if (delta2 && (!delta || !illm_dtype_ok(delta2_dt))) return ILLM_ERR_ARG;
    if (rows < 0 || E <= 0 || !illm_dtype_ok(w_dt) || !illm_dtype_ok(out_dt) ||
        (delta && (!illm_dtype_ok(delta_dt) || planes < 1 ||
                   (planes > 1 && E % 4 == 0 && plane_stride % 4))))
        return ILLM_ERR_ARG;
    if (rows == 0) return ILLM_OK;
    hipStream_t st = (hipStream_t)stream;
#define VEC(NV_, TH_)                                                                         \
    hipLaunchKernelGGL((add_rmsnorm_vec_kernel<NV_, TH_>), dim3(rows), dim3(TH_), 0, st, x,   \
                       delta, delta_dt, planes, plane_stride / 4, delta2, delta2_dt, w, w_dt, out,  \
                       out_dt, row_idx, E, eps, w2, out2)
    // few rows (decoding): wide blocks, one group of 4 floats per thread, to shorten the row's
    // critical path; many rows: narrow blocks so that more rows are in flight per CU
    if (E % 4 == 0 && rows <= 128 && E > 1024 && E <= 4096) VEC(1, 1024);
    else if (E % 4 == 0 && rows <= 128 && E > 4096 && E <= 8192) VEC(2, 1024);
    else if (E % 4 == 0 && E <= 1024) VEC(1, 256);
    else if (E % 4 == 0 && E <= 2048) VEC(2, 256);
    else if (E % 4 == 0 && E <= 4096) VEC(4, 256);
    else if (E % 4 == 0 && E <= 8192) VEC(8, 256);
    else
        hipLaunchKernelGGL(add_rmsnorm_kernel, dim3(rows), dim3(256), 0, st, x, delta, delta_dt,
                           planes, plane_stride, delta2, delta2_dt, w, w_dt, out, out_dt, row_idx, E,
                           eps, w2, out2);
#undef VEC
    return illm_launch_status();
}

extern "C" int illm_add2_rmsnorm(float* x, const void* delta, int delta_dt, int planes,
                                 size_t plane_stride, const void* delta2, int delta2_dt,
                                 const void* w, int w_dt, void* out, int out_dt,
                                 const int32_t* row_idx, int rows, int E, float eps, void* stream) {
    return illm_add2_rmsnorm_two(x, delta, delta_dt, planes, plane_stride, delta2, delta2_dt, w, nullptr,
                                 w_dt, out, nullptr, out_dt, row_idx, rows, E, eps, stream);
}

extern "C" int illm_add_rmsnorm(float* x, const void* delta, int delta_dt, int planes,
                                size_t plane_stride, const void* w, int w_dt, void* out,
                                int out_dt, const int32_t* row_idx, int rows, int E, float eps,
                                void* stream) {
    return illm_add2_rmsnorm(x, delta, delta_dt, planes, plane_stride, nullptr, 0, w, w_dt, out,
                             out_dt, row_idx, rows, E, eps, stream);
}

// ---------------------------------------------------------------- silu * up
__global__ void silu_mul_kernel(const void* __restrict__ gu, void* __restrict__ out, int dt,
                                int F) {
    const size_t t = blockIdx.y;
    const int f = blockIdx.x * blockDim.x + threadIdx.x;
    if (f >= F) return;
    const float g = ld_f(gu, dt, t * 2 * F + f);
    const float u = ld_f(gu, dt, t * 2 * F + F + f);
    st_f(out, dt, t * F + f, (g / (1.0f + expf(-g))) * u);
}

// bfloat16 rows with F % 8 == 0: 8 values (16 bytes) of gate and of up per thread
__global__ void __launch_bounds__(256)
silu_mul_bf16x8_kernel(const bf16_t* __restrict__ gu, bf16_t* __restrict__ out, int F) {
    const size_t t = blockIdx.y;
    const int f = (blockIdx.x * 256 + threadIdx.x) * 8;
    if (f >= F) return;
    const uint4 g = *(const uint4*)(gu + t * 2 * F + f);
    const uint4 u = *(const uint4*)(gu + t * 2 * F + F + f);
    const uint32_t gw[4] = {g.x, g.y, g.z, g.w}, uw[4] = {u.x, u.y, u.z, u.w};
    uint32_t ow[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const float g0 = __uint_as_float(gw[i] << 16), g1 = __uint_as_float(gw[i] & 0xffff0000u);
        const float u0 = __uint_as_float(uw[i] << 16), u1 = __uint_as_float(uw[i] & 0xffff0000u);
        const float r0 = (g0 / (1.0f + expf(-g0))) * u0, r1 = (g1 / (1.0f + expf(-g1))) * u1;
        ow[i] = pack_bf16x2(r0, r1);
    }
    *(uint4*)(out + t * F + f) = make_uint4(ow[0], ow[1], ow[2], ow[3]);
}

extern "C" int illm_silu_mul(const void* gate_up, void* out, int dt, int T, int F, void* stream) {
    if (T < 0 || F <= 0 || !illm_dtype_ok(dt)) return ILLM_ERR_ARG;
    if (T == 0) return ILLM_OK;
    if (dt == ILLM_BF16 && F % 8 == 0) {
        for (int t0 = 0; t0 < T; t0 += 65535) {
            const int rows = T - t0 < 65535 ? T - t0 : 65535;
            hipLaunchKernelGGL(silu_mul_bf16x8_kernel, dim3((F / 8 + 255) / 256, rows), dim3(256), 0,
                               (hipStream_t)stream, (const bf16_t*)gate_up + (size_t)t0 * 2 * F,
                               (bf16_t*)out + (size_t)t0 * F, F);
        }
        return illm_launch_status();
    }
    // gridDim.y is limited to 65535: rows beyond that go in further launches
    for (int t0 = 0; t0 < T; t0 += 65535) {
        const int rows = T - t0 < 65535 ? T - t0 : 65535;
        const size_t esz = dt == ILLM_BF16 ? 2 : 4;
        hipLaunchKernelGGL(silu_mul_kernel, dim3((F + 255) / 256, rows), dim3(256), 0,
                           (hipStream_t)stream,
                           (const void*)((const char*)gate_up + (size_t)t0 * 2 * F * esz),
                           (void*)((char*)out + (size_t)t0 * F * esz), dt, F);
    }
    return illm_launch_status();
}

// ---------------------------------------------------------------- rotation + cache store
// grid (T, nh + nkv): block (t, h) handles head h of row t; heads >= nh are k heads,
// whose block also stores the matching v head.  The angles come from a float32
// table that the host fills from double precision.
__global__ void rope_store_kernel(void* __restrict__ qkv, int dt,
                                  const float* __restrict__ cos_sin, int rot, int pairing,
                                  const int32_t* __restrict__ row_pos,
                                  const int32_t* __restrict__ row_slot,
                                  const int32_t* __restrict__ slot_len, void* __restrict__ kcache,
                                  void* __restrict__ vcache,
                                  const int32_t* __restrict__ page_table, int table_stride,
                                  int page_size, int ring, int nh, int nkv, int hd) {
    const int t = blockIdx.x, h = blockIdx.y;
    const int pos = row_pos[t];
    const size_t row = (size_t)t * (size_t)(nh + 2 * nkv) * hd;
    const size_t base = row + (size_t)h * hd;  // q heads, then k heads follow directly
    const int half = rot / 2;
    if (cos_sin) {
        const float* cs = cos_sin + (size_t)pos * rot;  // [rot/2][2]
        for (int i = threadIdx.x; i < half; i += blockDim.x) {
            const int a = pairing == 0 ? i : 2 * i;
            const int b = pairing == 0 ? i + hd / 2 : 2 * i + 1;  // partner at hd/2 (naive.cpp:393)
            const float c = cs[2 * i], s = cs[2 * i + 1];
            const float x0 = ld_f(qkv, dt, base + a), x1 = ld_f(qkv, dt, base + b);
            st_f(qkv, dt, base + a, x0 * c - x1 * s);
            st_f(qkv, dt, base + b, x0 * s + x1 * c);
        }
    }
    if (h < nh || kcache == nullptr) return;
    const int kvh = h - nh;
    const int slot = row_slot[t];
    if (ring > 0 && slot_len) {
        // a later row of this step lands on the same ring page: this one is already outside
        const int last_page = (slot_len[slot] - 1) / page_size;
        if (pos / page_size + ring <= last_page) return;
    }
    __syncthreads();  // the rotated k of this block is read back below
    const size_t dst = cache_row_offset(page_table, table_stride, slot, pos, page_size, ring, nkv,
                                        kvh, hd);
    const size_t vsrc = row + (size_t)(nh + nkv + kvh) * hd;
    const size_t esz = dt == ILLM_BF16 ? 2 : 4;
    if (esz == 2) {
        const bf16_t* ks = (const bf16_t*)qkv + base;
        const bf16_t* vs = (const bf16_t*)qkv + vsrc;
        bf16_t* kd = (bf16_t*)kcache + dst;
        bf16_t* vd = (bf16_t*)vcache + dst;
        for (int i = threadIdx.x; i < hd; i += blockDim.x) { kd[i] = ks[i]; vd[i] = vs[i]; }
    } else {
        const float* ks = (const float*)qkv + base;
        const float* vs = (const float*)qkv + vsrc;
        float* kd = (float*)kcache + dst;
        float* vd = (float*)vcache + dst;
        for (int i = threadIdx.x; i < hd; i += blockDim.x) { kd[i] = ks[i]; vd[i] = vs[i]; }
    }
}

// bfloat16, pairs (i, i + hd/2), all of the head rotated (rot == hd), hd % 16 == 0: one block
// per row; a thread rotates 8 pairs at a time with 16-byte loads, then the row's k and v
// heads are copied to the cache 16 bytes at a time.
__global__ void __launch_bounds__(256)
rope_store_bf16_kernel(bf16_t* __restrict__ qkv, const float* __restrict__ cos_sin,
                       const int32_t* __restrict__ row_pos, const int32_t* __restrict__ row_slot,
                       const int32_t* __restrict__ slot_len, bf16_t* __restrict__ kcache,
                       bf16_t* __restrict__ vcache, const int32_t* __restrict__ page_table,
                       int table_stride, int page_size, int ring, int nh, int nkv, int hd) {
    const int t = blockIdx.x;
    const int pos = row_pos[t];
    bf16_t* row = qkv + (size_t)t * (size_t)(nh + 2 * nkv) * hd;
    const int half = hd / 2, cpu8 = half / 8;             // chunks of 8 pairs per head
    if (cos_sin) {
        const float* cs = cos_sin + (size_t)pos * hd;     // [hd/2][2]
        for (int u = threadIdx.x; u < (nh + nkv) * cpu8; u += 256) {
            const int h = u / cpu8, i0 = (u - h * cpu8) * 8;
            bf16_t* p = row + (size_t)h * hd + i0;
            const uint4 a = *(const uint4*)p, b = *(const uint4*)(p + half);
            const uint32_t aw[4] = {a.x, a.y, a.z, a.w}, bw[4] = {b.x, b.y, b.z, b.w};
            uint32_t ao[4], bo[4];
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                const float4 c = *(const float4*)(cs + 2 * (i0 + 2 * j));   // cos, sin, cos, sin
                const float x0 = __uint_as_float(aw[j] << 16), x1 = __uint_as_float(aw[j] & 0xffff0000u);
                const float y0 = __uint_as_float(bw[j] << 16), y1 = __uint_as_float(bw[j] & 0xffff0000u);
                ao[j] = pack_bf16x2(x0 * c.x - y0 * c.y, x1 * c.z - y1 * c.w);
                bo[j] = pack_bf16x2(x0 * c.y + y0 * c.x, x1 * c.w + y1 * c.z);
            }
            *(uint4*)p = make_uint4(ao[0], ao[1], ao[2], ao[3]);
            *(uint4*)(p + half) = make_uint4(bo[0], bo[1], bo[2], bo[3]);
        }
    }
    if (kcache == nullptr) return;
    const int slot = row_slot[t];
    if (ring > 0 && slot_len) {
        const int last_page = (slot_len[slot] - 1) / page_size;
        if (pos / page_size + ring <= last_page) return;
    }
    __syncthreads();
    const int c8 = hd / 8;
    for (int u = threadIdx.x; u < 2 * nkv * c8; u += 256) {
        const int which = u / (nkv * c8), r = u - which * nkv * c8;
        const int kvh = r / c8, off = (r - kvh * c8) * 8;
        const size_t dst = cache_row_offset(page_table, table_stride, slot, pos, page_size, ring, nkv,
                                            kvh, hd) + off;
        const bf16_t* src = row + (size_t)(nh + which * nkv + kvh) * hd + off;
        *(uint4*)((which ? vcache : kcache) + dst) = *(const uint4*)src;
    }
}

extern "C" int illm_rope_store(void* qkv, int dt, const float* cos_sin, int max_pos, int rot,
                               int pairing, const int32_t* row_pos, const int32_t* row_slot,
                               const int32_t* slot_len, void* kcache, void* vcache,
                               const int32_t* page_table, int table_stride, int page_size,
                               int ring, int T, int nh, int nkv, int hd, void* stream) {
    if (T < 0 || nh <= 0 || nkv < 0 || hd <= 0 || !illm_dtype_ok(dt)) return ILLM_ERR_ARG;
    if (cos_sin && (rot <= 0 || rot > hd || (rot & 1) || max_pos <= 0)) return ILLM_ERR_ARG;
    if (pairing != 0 && pairing != 1) return ILLM_ERR_ARG;
    if (kcache && (!vcache || !page_table || !row_slot || page_size <= 0 || table_stride <= 0))
        return ILLM_ERR_ARG;
    if (nh + nkv > 65535) return ILLM_ERR_ARG;
    if (T == 0) return ILLM_OK;
    if (dt == ILLM_BF16 && hd % 16 == 0 && (!cos_sin || (pairing == 0 && rot == hd))) {
        hipLaunchKernelGGL(rope_store_bf16_kernel, dim3(T), dim3(256), 0, (hipStream_t)stream,
                           (bf16_t*)qkv, cos_sin, row_pos, row_slot, slot_len, (bf16_t*)kcache,
                           (bf16_t*)vcache, page_table, table_stride, page_size, ring, nh, nkv, hd);
        return illm_launch_status();
    }
    hipLaunchKernelGGL(rope_store_kernel, dim3(T, nh + nkv), dim3(64), 0, (hipStream_t)stream, qkv,
                       dt, cos_sin, rot, pairing, row_pos, row_slot, slot_len, kcache, vcache,
                       page_table, table_stride, page_size, ring, nh, nkv, hd);
    return illm_launch_status();
}

extern "C" int illm_version() { return 1; }
