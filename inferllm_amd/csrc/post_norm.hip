// Residual streams whose sublayers are normed behind and not in front: what stands between one
// sublayer's output and the next sublayer's input, in one pass over the row.
//     x   <- x + gain * post(a)                       (a null: nothing is added)
//     out  = the row itself or a norm of it, in the output's type
// post and the output's norm are each one of: none, the RMS norm v / sqrt(mean(v^2) + eps) * w, the layer
// norm (v - mean) / sqrt(mean((v - mean)^2) + eps) * w + b (b null: none).  With `row_idx` only those rows
// are formed and x is left as it is.  Everything but the stored rows is float32; a row's sums run in
// an order that its width alone fixes.
#include "api.h"
#include "common.h"

// (mean, scale) of a row whose entries a thread holds in v (those beyond the row are 0 and not `in`)
template <int N>
__device__ __forceinline__ float2 row_stats(const float* v, const bool* in, int kind, int E, float eps, float* red) {
    float mean = 0.f;
    if (kind == ILLM_NORM_LAYER) {
        float s = 0.f;
#pragma unroll
        for (int k = 0; k < N; ++k) s += v[k];
        mean = block_sum(s, red) / (float)E;
    }
    float ss = 0.f;
#pragma unroll
    for (int k = 0; k < N; ++k) {
        const float d = in[k / 4] ? v[k] - mean : 0.f;
        ss = fmaf(d, d, ss);
    }
    ss = block_sum(ss, red);
    return make_float2(mean, 1.0f / sqrtf(ss / (float)E + eps));
}

// grid (rows); 256 threads.  A thread owns NV groups of 4 consecutive columns (E % 4 == 0, E <= 1024 NV)
// and asks for all it reads before it uses any of it.
template <int NV>
__global__ void __launch_bounds__(256)
post_add_norm_kernel(float* __restrict__ x, const void* __restrict__ a, int a_dt, int post_kind,
                     const void* __restrict__ pw, const void* __restrict__ pb, int pw_dt, float post_eps,
                     float gain, int out_kind, const void* __restrict__ w, const void* __restrict__ b, int w_dt,
                     float eps, void* __restrict__ out, int out_dt, const int32_t* __restrict__ row_idx, int E) {
    __shared__ float red[16];
    const int r = blockIdx.x, n4 = E / 4;
    const size_t ib4 = (size_t)(row_idx ? row_idx[r] : r) * n4, ob4 = (size_t)r * n4;
    const float4 zero4 = make_float4(0.f, 0.f, 0.f, 0.f);
    float4 xv[NV], av[NV], pwv[NV], pbv[NV], wv[NV], bv[NV];
    bool in[NV];
#pragma unroll
    for (int k = 0; k < NV; ++k) {
        const int i = threadIdx.x + 256 * k;
        in[k] = i < n4;
        xv[k] = in[k] ? ((const float4*)x)[ib4 + i] : zero4;
        av[k] = (a && in[k]) ? ld_f4(a, a_dt, ib4 + i) : zero4;
        pwv[k] = (a && post_kind && in[k]) ? ld_f4(pw, pw_dt, i) : zero4;
        pbv[k] = (a && pb && in[k]) ? ld_f4(pb, pw_dt, i) : zero4;
        wv[k] = (out_kind && in[k]) ? ld_f4(w, w_dt, i) : zero4;
        bv[k] = (out_kind && b && in[k]) ? ld_f4(b, w_dt, i) : zero4;
    }
    if (a) {
        float2 st = make_float2(0.f, 1.f);
        if (post_kind) st = row_stats<4 * NV>((const float*)av, in, post_kind, E, post_eps, red);
#pragma unroll
        for (int k = 0; k < NV; ++k) {
            const int i = threadIdx.x + 256 * k;
            if (!in[k]) continue;
            if (post_kind) {
                av[k].x = (av[k].x - st.x) * st.y * pwv[k].x + pbv[k].x;
                av[k].y = (av[k].y - st.x) * st.y * pwv[k].y + pbv[k].y;
                av[k].z = (av[k].z - st.x) * st.y * pwv[k].z + pbv[k].z;
                av[k].w = (av[k].w - st.x) * st.y * pwv[k].w + pbv[k].w;
            }
            xv[k].x += gain * av[k].x; xv[k].y += gain * av[k].y;
            xv[k].z += gain * av[k].z; xv[k].w += gain * av[k].w;
            if (!row_idx) ((float4*)x)[ib4 + i] = xv[k];
        }
    }
    if (!out) return;
    float2 st = make_float2(0.f, 1.f);
    if (out_kind) st = row_stats<4 * NV>((const float*)xv, in, out_kind, E, eps, red);
#pragma unroll
    for (int k = 0; k < NV; ++k) {
        const int i = threadIdx.x + 256 * k;
        if (!in[k]) continue;
        float4 y = xv[k];
        if (out_kind) {
            y.x = (y.x - st.x) * st.y * wv[k].x + bv[k].x;
            y.y = (y.y - st.x) * st.y * wv[k].y + bv[k].y;
            y.z = (y.z - st.x) * st.y * wv[k].z + bv[k].z;
            y.w = (y.w - st.x) * st.y * wv[k].w + bv[k].w;
        }
        st_f4(out, out_dt, ob4 + i, y);
    }
}

// Any width: the row stays in LDS (E floats) between the passes.
__global__ void __launch_bounds__(256)
post_add_norm_any_kernel(float* __restrict__ x, const void* __restrict__ a, int a_dt, int post_kind,
                         const void* __restrict__ pw, const void* __restrict__ pb, int pw_dt, float post_eps,
                         float gain, int out_kind, const void* __restrict__ w, const void* __restrict__ b,
                         int w_dt, float eps, void* __restrict__ out, int out_dt,
                         const int32_t* __restrict__ row_idx, int E) {
    extern __shared__ float row[];
    __shared__ float red[16];
    const int r = blockIdx.x;
    const size_t ib = (size_t)(row_idx ? row_idx[r] : r) * E, ob = (size_t)r * E;
    auto stats = [&](int kind, float e) {
        float mean = 0.f, s = 0.f;
        if (kind == ILLM_NORM_LAYER) {
            for (int i = threadIdx.x; i < E; i += 256) s += row[i];
            mean = block_sum(s, red) / (float)E;
        }
        s = 0.f;
        for (int i = threadIdx.x; i < E; i += 256) s = fmaf(row[i] - mean, row[i] - mean, s);
        s = block_sum(s, red);
        return make_float2(mean, 1.0f / sqrtf(s / (float)E + e));
    };
    // (a thread reads and writes its own entries of `row` only)
    float2 st = make_float2(0.f, 1.f);
    if (a) {
        for (int i = threadIdx.x; i < E; i += 256) row[i] = ld_f(a, a_dt, ib + i);
        if (post_kind) st = stats(post_kind, post_eps);
    }
    for (int i = threadIdx.x; i < E; i += 256) {
        float v = x[ib + i];
        if (a) {
            float y = row[i];
            if (post_kind) y = (y - st.x) * st.y * ld_f(pw, pw_dt, i) + (pb ? ld_f(pb, pw_dt, i) : 0.f);
            v += gain * y;
            if (!row_idx) x[ib + i] = v;
        }
        row[i] = v;
    }
    if (!out) return;
    if (out_kind) st = stats(out_kind, eps);
    for (int i = threadIdx.x; i < E; i += 256) {
        float y = row[i];
        if (out_kind) y = (y - st.x) * st.y * ld_f(w, w_dt, i) + (b ? ld_f(b, w_dt, i) : 0.f);
        st_f(out, out_dt, ob + i, y);
    }
}

extern "C" int illm_post_add_norm(float* x, const void* a, int a_dt, int post_kind, const void* pw, const void* pb,
                                  int pw_dt, float post_eps, float gain, int out_kind, const void* w,
                                  const void* b, int w_dt, float eps, void* out, int out_dt,
                                  const int32_t* row_idx, int rows, int E, void* stream) {
    auto known = [](int k) { return k == ILLM_NORM_NONE || k == ILLM_NORM_RMS || k == ILLM_NORM_LAYER; };
    if (rows < 0 || E <= 0 || !known(post_kind) || !known(out_kind) || (a && !illm_dtype_ok(a_dt)) ||
        (a && post_kind && (!pw || !illm_dtype_ok(pw_dt))) || (out && !illm_dtype_ok(out_dt)) ||
        (out && out_kind && (!w || !illm_dtype_ok(w_dt))) || (pb && post_kind != ILLM_NORM_LAYER) ||
        (b && out_kind != ILLM_NORM_LAYER) || (row_idx && !out))
        return ILLM_ERR_ARG;
    if (rows == 0 || (!a && !out)) return ILLM_OK;
    hipStream_t st = (hipStream_t)stream;
#define GO(KERNEL_, LDS_)                                                                                  \
    hipLaunchKernelGGL(KERNEL_, dim3(rows), dim3(256), LDS_, st, x, a, a_dt, post_kind, pw, pb, pw_dt, post_eps, \
                       gain, out_kind, w, b, w_dt, eps, out, out_dt, row_idx, E)
    if (E % 4 == 0 && E <= 8192) {
        if (E <= 1024) GO((post_add_norm_kernel<1>), 0);
        else if (E <= 2048) GO((post_add_norm_kernel<2>), 0);
        else if (E <= 4096) GO((post_add_norm_kernel<4>), 0);
        else GO((post_add_norm_kernel<8>), 0);
        return illm_launch_status();
    }
    const size_t lds = (size_t)E * sizeof(float);
    if (lds > 64 * 1024 - 256) return ILLM_ERR_ARG;
    if (lds > 48 * 1024 &&
        hipFuncSetAttribute((const void*)post_add_norm_any_kernel, hipFuncAttributeMaxDynamicSharedMemorySize,
                            (int)lds) != hipSuccess)
        return ILLM_ERR_LAUNCH;
    GO(post_add_norm_any_kernel, lds);
#undef GO
    return illm_launch_status();
}
