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

// ---------------------------------------------------------------- the same pass for two outputs side by side,
// the embedding's rows and a token shift
//     y  = a,  or of two sublayers side by side  y = pair_scale (rms(a) aw + rms(b) bw)       (b given)
//     x <- x + gain rms(y) pw + plus                                            (a null: x + plus; plus null: 0)
//     h  = rms(x) w, rounded to the output's type
//     out = h,  or S mixes with the row of the token before, out[s] = h + (h_before - h) mu_s           (mu given)
// rms(v) = v / sqrt(mean(v^2) + eps) with an eps each.  The mixes are for steps of one row a sequence: h_before is
// tail [slots][E], which takes h.  With `row_idx` only those rows are formed and x is left as it is.
// grid (rows); 256 threads, NV groups of 4 columns a thread; NV 0: any width, two rows of E floats in LDS.
struct PostMix {
    float* x;
    const void *a, *b, *aw, *bw, *pw, *w;
    const float *plus, *mu;
    void *out, *tail;
    const int32_t *row_idx, *row_slot;
    int a_dt, b_dt, pair_dt, pw_dt, w_dt, out_dt, tail_dt, E, S, rows;
    float pair_eps, pair_scale, post_eps, gain, eps;
};

__device__ __forceinline__ float2 block_sum2(float u, float v, float* red) {
    const int lane = threadIdx.x & (ILLM_WAVE - 1), w = threadIdx.x / ILLM_WAVE;
    u = wave_sum(u); v = wave_sum(v);
    __syncthreads();
    if (lane == 0) { red[w] = u; red[8 + w] = v; }
    __syncthreads();
    return make_float2((red[0] + red[1]) + (red[2] + red[3]), (red[8] + red[9]) + (red[10] + red[11]));
}
__device__ __forceinline__ float sum_sq(const float4 v) { return (v.x * v.x + v.y * v.y) + (v.z * v.z + v.w * v.w); }

#define POST_MIX_AHEAD 5   // mixes whose weights are asked for with the row (rows of up to 2,048 columns)

template <int NV, bool PAIR, bool SHIFT>
__global__ void __launch_bounds__(256)
post_mix_norm_kernel(PostMix m) {
    extern __shared__ float row[];
    __shared__ float red[16];
    const int r = blockIdx.x, E = m.E;
    const size_t in_row = m.row_idx ? m.row_idx[r] : r;
    const int slot = SHIFT ? m.row_slot[r] : 0;
    if (NV > 0) {
        const int n4 = E / 4;
        const size_t ib = in_row * n4, ob = (size_t)r * n4;
        const float4 zero4 = make_float4(0.f, 0.f, 0.f, 0.f);
        float4 x[NV ? NV : 1], a[NV ? NV : 1], b[NV && PAIR ? NV : 1], aw[NV && PAIR ? NV : 1], bw[NV && PAIR ? NV : 1];
        float4 pw[NV ? NV : 1], w[NV ? NV : 1], pl[NV ? NV : 1], old[NV && SHIFT ? NV : 1];
        constexpr bool AHEAD = SHIFT && NV > 0 && NV <= 2;
        float4 mu[AHEAD ? NV : 1][AHEAD ? POST_MIX_AHEAD : 1];
#pragma unroll
        for (int k = 0; k < NV; ++k) {
            const int i = threadIdx.x + 256 * k;
            const bool in = i < n4;
            x[k] = in ? ((const float4*)m.x)[ib + i] : zero4;
            a[k] = (m.a && in) ? ld_f4(m.a, m.a_dt, ib + i) : zero4;
            if (PAIR) {
                b[k] = in ? ld_f4(m.b, m.b_dt, ib + i) : zero4;
                aw[k] = in ? ld_f4(m.aw, m.pair_dt, i) : zero4;
                bw[k] = in ? ld_f4(m.bw, m.pair_dt, i) : zero4;
            }
            pw[k] = (m.a && in) ? ld_f4(m.pw, m.pw_dt, i) : zero4;
            pl[k] = (m.plus && in) ? ((const float4*)m.plus)[ib + i] : zero4;
            w[k] = in ? ld_f4(m.w, m.w_dt, i) : zero4;
            if (AHEAD) {
#pragma unroll
                for (int s = 0; s < POST_MIX_AHEAD; ++s)
                    if (s < m.S) mu[k][s] = in ? ((const float4*)m.mu)[(size_t)s * n4 + i] : zero4;
            }
            if (SHIFT) old[k] = in ? ld_f4(m.tail, m.tail_dt, (size_t)slot * n4 + i) : zero4;
        }
        if (m.a) {
            if (PAIR) {
                float sa = 0.f, sb = 0.f;
#pragma unroll
                for (int k = 0; k < NV; ++k) { sa += sum_sq(a[k]); sb += sum_sq(b[k]); }
                const float2 s = block_sum2(sa, sb, red);
                const float ia = 1.0f / sqrtf(s.x / (float)E + m.pair_eps), ib2 = 1.0f / sqrtf(s.y / (float)E + m.pair_eps);
#pragma unroll
                for (int k = 0; k < NV; ++k) {
                    a[k].x = m.pair_scale * (a[k].x * ia * aw[k].x + b[k].x * ib2 * bw[k].x);
                    a[k].y = m.pair_scale * (a[k].y * ia * aw[k].y + b[k].y * ib2 * bw[k].y);
                    a[k].z = m.pair_scale * (a[k].z * ia * aw[k].z + b[k].z * ib2 * bw[k].z);
                    a[k].w = m.pair_scale * (a[k].w * ia * aw[k].w + b[k].w * ib2 * bw[k].w);
                }
            }
            float ss = 0.f;
#pragma unroll
            for (int k = 0; k < NV; ++k) ss += sum_sq(a[k]);
            ss = block_sum(ss, red);
            const float inv = 1.0f / sqrtf(ss / (float)E + m.post_eps);
#pragma unroll
            for (int k = 0; k < NV; ++k) {
                x[k].x += m.gain * (a[k].x * inv * pw[k].x);
                x[k].y += m.gain * (a[k].y * inv * pw[k].y);
                x[k].z += m.gain * (a[k].z * inv * pw[k].z);
                x[k].w += m.gain * (a[k].w * inv * pw[k].w);
            }
        }
        float ss = 0.f;
#pragma unroll
        for (int k = 0; k < NV; ++k) {
            const int i = threadIdx.x + 256 * k;
            x[k].x += pl[k].x; x[k].y += pl[k].y; x[k].z += pl[k].z; x[k].w += pl[k].w;
            if (!m.row_idx && (m.a || m.plus) && i < n4) ((float4*)m.x)[ib + i] = x[k];
            ss += sum_sq(x[k]);
        }
        ss = block_sum(ss, red);
        const float inv = 1.0f / sqrtf(ss / (float)E + m.eps);
#pragma unroll
        for (int k = 0; k < NV; ++k) {
            const int i = threadIdx.x + 256 * k;
            if (i >= n4) continue;
            float4 h = make_float4((x[k].x * inv) * w[k].x, (x[k].y * inv) * w[k].y, (x[k].z * inv) * w[k].z,
                                   (x[k].w * inv) * w[k].w);
            if (!SHIFT) {
                st_f4(m.out, m.out_dt, ob + i, h);
                continue;
            }
            if (m.out_dt == ILLM_BF16) {
                h.x = bf16_to_f32(f32_to_bf16(h.x)); h.y = bf16_to_f32(f32_to_bf16(h.y));
                h.z = bf16_to_f32(f32_to_bf16(h.z)); h.w = bf16_to_f32(f32_to_bf16(h.w));
            }
            const float4 d = make_float4(old[k].x - h.x, old[k].y - h.y, old[k].z - h.z, old[k].w - h.w);
            auto mix = [&](int s, const float4 u) __attribute__((always_inline)) {
                st_f4(m.out, m.out_dt, ((size_t)s * m.rows) * n4 + ob + i,
                      make_float4(fmaf(d.x, u.x, h.x), fmaf(d.y, u.y, h.y), fmaf(d.z, u.z, h.z), fmaf(d.w, u.w, h.w)));
            };
            if (AHEAD) {
#pragma unroll
                for (int s = 0; s < POST_MIX_AHEAD; ++s)
                    if (s < m.S) mix(s, mu[k][s]);
            }
            for (int s = AHEAD ? POST_MIX_AHEAD : 0; s < m.S; ++s) mix(s, ((const float4*)m.mu)[(size_t)s * n4 + i]);
            st_f4(m.tail, m.tail_dt, (size_t)slot * n4 + i, h);
        }
        return;
    }
    const size_t ib = in_row * E, ob = (size_t)r * E;
    float* y = row + E;
    // (a thread reads and writes its own entries of the rows in LDS only)
    float inv = 0.f;
    if (m.a) {
        if (PAIR) {
            float sa = 0.f, sb = 0.f;
            for (int i = threadIdx.x; i < E; i += 256) {
                const float u = ld_f(m.a, m.a_dt, ib + i), v = ld_f(m.b, m.b_dt, ib + i);
                sa = fmaf(u, u, sa); sb = fmaf(v, v, sb);
            }
            const float2 s = block_sum2(sa, sb, red);
            const float ia = 1.0f / sqrtf(s.x / (float)E + m.pair_eps), ib2 = 1.0f / sqrtf(s.y / (float)E + m.pair_eps);
            for (int i = threadIdx.x; i < E; i += 256)
                y[i] = m.pair_scale * (ld_f(m.a, m.a_dt, ib + i) * ia * ld_f(m.aw, m.pair_dt, i) +
                                       ld_f(m.b, m.b_dt, ib + i) * ib2 * ld_f(m.bw, m.pair_dt, i));
        } else {
            for (int i = threadIdx.x; i < E; i += 256) y[i] = ld_f(m.a, m.a_dt, ib + i);
        }
        float ss = 0.f;
        for (int i = threadIdx.x; i < E; i += 256) ss = fmaf(y[i], y[i], ss);
        ss = block_sum(ss, red);
        inv = 1.0f / sqrtf(ss / (float)E + m.post_eps);
    }
    float ss = 0.f;
    for (int i = threadIdx.x; i < E; i += 256) {
        float v = m.x[ib + i];
        if (m.a) v += m.gain * (y[i] * inv * ld_f(m.pw, m.pw_dt, i));
        if (m.plus) v += m.plus[ib + i];
        if (!m.row_idx && (m.a || m.plus)) m.x[ib + i] = v;
        row[i] = v;
        ss = fmaf(v, v, ss);
    }
    ss = block_sum(ss, red);
    inv = 1.0f / sqrtf(ss / (float)E + m.eps);
    for (int i = threadIdx.x; i < E; i += 256) {
        float h = (row[i] * inv) * ld_f(m.w, m.w_dt, i);
        if (!SHIFT) {
            st_f(m.out, m.out_dt, ob + i, h);
            continue;
        }
        if (m.out_dt == ILLM_BF16) h = bf16_to_f32(f32_to_bf16(h));
        const float d = ld_f(m.tail, m.tail_dt, (size_t)slot * E + i) - h;
        for (int s = 0; s < m.S; ++s)
            st_f(m.out, m.out_dt, (size_t)s * m.rows * E + ob + i, fmaf(d, m.mu[(size_t)s * E + i], h));
        st_f(m.tail, m.tail_dt, (size_t)slot * E + i, h);
    }
}

extern "C" int illm_post_mix_norm(float* x, const void* a, int a_dt, const void* b, int b_dt, const void* aw,
                                  const void* bw, int pair_dt, float pair_eps, float pair_scale, const void* pw,
                                  int pw_dt, float post_eps, float gain, const float* plus, const void* w, int w_dt,
                                  float eps, void* out, int out_dt, const float* mu, int S, void* tail, int tail_dt,
                                  const int32_t* row_slot, const int32_t* row_idx, int rows, int E, void* stream) {
    if (rows < 0 || E <= 0 || !x || !w || !out || !illm_dtype_ok(w_dt) || !illm_dtype_ok(out_dt) ||
        (a && (!illm_dtype_ok(a_dt) || !pw || !illm_dtype_ok(pw_dt))) ||
        (b && (!a || !aw || !bw || !illm_dtype_ok(b_dt) || !illm_dtype_ok(pair_dt))) ||
        (mu && (S <= 0 || !tail || !row_slot || row_idx || !illm_dtype_ok(tail_dt))))
        return ILLM_ERR_ARG;
    if (rows == 0) return ILLM_OK;
    hipStream_t st = (hipStream_t)stream;
    PostMix m = {x, a, b, aw, bw, pw, w, plus, mu, out, tail, row_idx, row_slot, a_dt, b_dt, pair_dt, pw_dt, w_dt,
                 out_dt, tail_dt, E, S, rows, pair_eps, pair_scale, post_eps, gain, eps};
#define GO(NV_, P_, S_, LDS_) hipLaunchKernelGGL((post_mix_norm_kernel<NV_, P_, S_>), dim3(rows), dim3(256), LDS_, st, m)
#define GO_F(NV_, LDS_)                                                                                    \
    do {                                                                                                   \
        if (b && mu) GO(NV_, true, true, LDS_);                                                            \
        else if (b) GO(NV_, true, false, LDS_);                                                            \
        else if (mu) GO(NV_, false, true, LDS_);                                                           \
        else GO(NV_, false, false, LDS_);                                                                  \
    } while (0)
    if (E % 4 == 0 && E <= 8192) {
        if (E <= 1024) GO_F(1, 0);
        else if (E <= 2048) GO_F(2, 0);
        else if (E <= 4096) GO_F(4, 0);
        else GO_F(8, 0);
        return illm_launch_status();
    }
    const size_t lds = (size_t)2 * E * sizeof(float);
    if (lds > 48 * 1024) return ILLM_ERR_ARG;
    GO_F(0, lds);
#undef GO_F
#undef GO
    return illm_launch_status();
}
