// Four linear mixers with a matrix of state S [key dim, value dim] (float32) per head and no convolution:
//
// Lightning attention, one fixed decay lam a head: q, k, v through SiLU,
//     S <- lam S + k v^T;   o = S^T q
//   lightning_prepare   the inputs of illm_gated_scan as float32 (any number of rows)
//   lightning_step      single tokens: SiLU, the state's update and o in one launch
//   lightning_chunks    long steps, chunks of FD_CHUNK tokens in parallel (three launches, see below)
//
// The delta rule with a removal vector, one decay w and one rate a per key channel, u = k / |k|:
//     w = exp(-rate sigmoid(z + w0)),  a = sigmoid(y + a_bias),   S <- diag(w) S - (a u)(u^T S) + k v^T;   o = S^T r
//   removal_prepare     the inputs of illm_gated_scan (with `removal`) as float32
//   removal_step        single tokens in one launch, z = W2 tanh(y1) of the low-rank map included
//
// Retention, one fixed decay lam a head, q and k turned by their positions (pairs i, i + rot / 2) and k
// times dk^-1/2, neither activated:  S <- lam S + k v^T;   o = S^T q
//   retention_prepare   q, k (and, for illm_gated_scan, the rest of its inputs) as float32
//   retention_step      single tokens: rotation, the state's update and o in one launch
//   retention_chunks    long steps, as lightning_chunks
//
// Time mixing with a decay w a key channel and a bonus u for the current token, w = exp(-exp(z + w0)):
//     o = (S + diag(u) k v^T)^T r;   S <- diag(w) S + k v^T
//   time_mix_step       single tokens in one launch, z = W2 tanh(y1) included (long steps: time_mix.hip)
//
// Behind any: group_norm_gate, o RMS-normed in equal parts of the row, a weight of the row's width, a
// gate.  Everything but the stored projections is float32.  A sequence's rows in a step are consecutive.
#include <math.h>

#include "api.h"
#include "common.h"

__device__ __forceinline__ float fd_sigmoid(float x) { return 1.0f / (1.0f + expf(-x)); }
__device__ __forceinline__ float fd_silu(float x) { return x / (1.0f + expf(-x)); }

// ---------------------------------------------------------------- inputs of the scan
// grid (rows); 256 threads.  U [T, u_stride]: q at q_off and k at k_off (H dk), v at v_off (H dv).
__global__ void __launch_bounds__(256)
lightning_prepare_kernel(const void* __restrict__ U, int dt, int u_stride, int q_off, int k_off, int v_off,
                         const float* __restrict__ decay, float* __restrict__ qn, float* __restrict__ kn,
                         float* __restrict__ vv, float* __restrict__ beta, float* __restrict__ dec, int H,
                         int dk, int dv) {
    const size_t t = blockIdx.x, u0 = t * u_stride;
    for (int e = threadIdx.x; e < H * dk; e += 256) {
        qn[t * H * dk + e] = fd_silu(ld_f(U, dt, u0 + q_off + e));
        kn[t * H * dk + e] = fd_silu(ld_f(U, dt, u0 + k_off + e));
    }
    for (int e = threadIdx.x; e < H * dv; e += 256) vv[t * H * dv + e] = fd_silu(ld_f(U, dt, u0 + v_off + e));
    for (int e = threadIdx.x; e < H; e += 256) { beta[t * H + e] = 1.0f; dec[t * H + e] = decay[e]; }
}

static bool fd_columns_ok(int u_stride, int off, int n) { return off >= 0 && off + n <= u_stride; }

extern "C" int illm_lightning_prepare(const void* U, int dt, int u_stride, int q_off, int k_off, int v_off,
                                      const float* decay, float* qn, float* kn, float* vv, float* beta,
                                      float* dec, int T, int H, int dk, int dv, void* stream) {
    if (T < 0 || H <= 0 || dk <= 0 || dv <= 0 || !illm_dtype_ok(dt) || !fd_columns_ok(u_stride, q_off, H * dk) ||
        !fd_columns_ok(u_stride, k_off, H * dk) || !fd_columns_ok(u_stride, v_off, H * dv))
        return ILLM_ERR_ARG;
    if (T == 0) return ILLM_OK;
    hipLaunchKernelGGL(lightning_prepare_kernel, dim3(T), dim3(256), 0, (hipStream_t)stream, U, dt, u_stride,
                       q_off, k_off, v_off, decay, qn, kn, vv, beta, dec, H, dk, dv);
    return illm_launch_status();
}

// grid (rows); 256 threads.  q and k heads turned by the row's position and k times k_scale; vv, beta and
// dec may be null (the chunks take v and the decays as they are).
__global__ void __launch_bounds__(256)
retention_prepare_kernel(const void* __restrict__ U, int dt, int u_stride, int q_off, int k_off, int v_off,
                         const float* __restrict__ decay, const float* __restrict__ cos_sin, int rot, float k_scale,
                         const int32_t* __restrict__ row_pos, float* __restrict__ qn, float* __restrict__ kn,
                         float* __restrict__ vv, float* __restrict__ beta, float* __restrict__ dec, int H,
                         int dk, int dv) {
    const size_t t = blockIdx.x, u0 = t * u_stride;
    const float* cs = rot > 0 ? cos_sin + (size_t)row_pos[t] * rot : nullptr;
    const int half = rot / 2;
    const bool quads = dk % 4 == 0 && half % 4 == 0 && u_stride % 4 == 0 && q_off % 4 == 0 && k_off % 4 == 0;
    // four neighbouring pairs (or dims beyond the rotation) of a head at a time
    for (int e4 = threadIdx.x; quads && e4 < H * dk / 4; e4 += 256) {
        const int e = 4 * e4, i = e % dk;
        if (i >= half && i < rot) continue;              // (the partners, brought along by the first of a pair)
        const size_t at = t * H * dk + e;
        float4 q = ld_f4(U, dt, (u0 + q_off + e) / 4), k = ld_f4(U, dt, (u0 + k_off + e) / 4);
        if (i < rot) {
            const float4 q2 = ld_f4(U, dt, (u0 + q_off + e + half) / 4), k2 = ld_f4(U, dt, (u0 + k_off + e + half) / 4);
            const float4 c0 = *(const float4*)(cs + 2 * i), c1 = *(const float4*)(cs + 2 * i + 4);   // c s c s
            *(float4*)(qn + at + half) = make_float4(q2.x * c0.x + q.x * c0.y, q2.y * c0.z + q.y * c0.w,
                                                     q2.z * c1.x + q.z * c1.y, q2.w * c1.z + q.w * c1.w);
            *(float4*)(kn + at + half) =
                make_float4((k2.x * c0.x + k.x * c0.y) * k_scale, (k2.y * c0.z + k.y * c0.w) * k_scale,
                            (k2.z * c1.x + k.z * c1.y) * k_scale, (k2.w * c1.z + k.w * c1.w) * k_scale);
            q = make_float4(q.x * c0.x - q2.x * c0.y, q.y * c0.z - q2.y * c0.w, q.z * c1.x - q2.z * c1.y,
                            q.w * c1.z - q2.w * c1.w);
            k = make_float4(k.x * c0.x - k2.x * c0.y, k.y * c0.z - k2.y * c0.w, k.z * c1.x - k2.z * c1.y,
                            k.w * c1.z - k2.w * c1.w);
        }
        *(float4*)(qn + at) = q;
        *(float4*)(kn + at) = make_float4(k.x * k_scale, k.y * k_scale, k.z * k_scale, k.w * k_scale);
    }
    for (int e = threadIdx.x; !quads && e < H * dk; e += 256) {
        const int i = e % dk;
        float q = ld_f(U, dt, u0 + q_off + e), k = ld_f(U, dt, u0 + k_off + e);
        if (i < rot) {
            const int j = i < half ? i : i - half, other = e + (i < half ? half : -half);
            const float c = cs[2 * j], sn = i < half ? -cs[2 * j + 1] : cs[2 * j + 1];
            q = q * c + ld_f(U, dt, u0 + q_off + other) * sn;
            k = k * c + ld_f(U, dt, u0 + k_off + other) * sn;
        }
        qn[t * H * dk + e] = q;
        kn[t * H * dk + e] = k * k_scale;
    }
    if (vv)
        for (int e = threadIdx.x; e < H * dv; e += 256) vv[t * H * dv + e] = ld_f(U, dt, u0 + v_off + e);
    if (beta)
        for (int e = threadIdx.x; e < H; e += 256) { beta[t * H + e] = 1.0f; dec[t * H + e] = decay[e]; }
}

extern "C" int illm_retention_prepare(const void* U, int dt, int u_stride, int q_off, int k_off, int v_off,
                                      const float* decay, const float* cos_sin, int n_positions, int rot, float k_scale,
                                      const int32_t* row_pos, float* qn, float* kn, float* vv, float* beta,
                                      float* dec, int T, int H, int dk, int dv, void* stream) {
    if (T < 0 || H <= 0 || dk <= 0 || dv <= 0 || !illm_dtype_ok(dt) || rot < 0 || rot % 2 || rot > dk ||
        (rot > 0 && (!cos_sin || n_positions <= 0 || !row_pos)) || !fd_columns_ok(u_stride, q_off, H * dk) ||
        !fd_columns_ok(u_stride, k_off, H * dk) || !fd_columns_ok(u_stride, v_off, H * dv) || (!beta) != (!dec))
        return ILLM_ERR_ARG;
    if (T == 0) return ILLM_OK;
    hipLaunchKernelGGL(retention_prepare_kernel, dim3(T), dim3(256), 0, (hipStream_t)stream, U, dt, u_stride, q_off,
                       k_off, v_off, decay, cos_sin, rot, k_scale, row_pos, qn, kn, vv, beta, dec, H, dk, dv);
    return illm_launch_status();
}

// grid (rows, ceil(H / 4)); a wave takes a head, lanes over its d channels (d <= 256).  U: r, k, v at
// r_off, k_off, v_off and the rates' pre-activations at a_off, all H d wide; Z [T, z_stride] (H d wide).
#define FD_VEC 4
__global__ void __launch_bounds__(256)
removal_prepare_kernel(const void* __restrict__ U, int dt, int u_stride, int r_off, int k_off, int v_off,
                       int a_off, const float* __restrict__ a_bias, const void* __restrict__ Z, int z_dt,
                       int z_stride, const float* __restrict__ w0, float rate, float* __restrict__ qn,
                       float* __restrict__ kn, float* __restrict__ vv, float* __restrict__ beta,
                       float* __restrict__ dec, float* __restrict__ removal, int H, int d) {
    const size_t t = blockIdx.x, u0 = t * u_stride;
    const int h = blockIdx.y * 4 + wave_index(), lane = threadIdx.x & 63;
    if (h >= H) return;
    float k[FD_VEC], ss = 0.f;
#pragma unroll
    for (int e = 0; e < FD_VEC; ++e) {
        const int i = lane + 64 * e;
        k[e] = i < d ? ld_f(U, dt, u0 + k_off + h * d + i) : 0.f;
        ss = fmaf(k[e], k[e], ss);
    }
    const float inv = 1.0f / sqrtf(wave_sum(ss) + 1e-6f);
    if (lane == 0) beta[t * H + h] = inv;
#pragma unroll
    for (int e = 0; e < FD_VEC; ++e) {
        const int i = lane + 64 * e, c = h * d + i;
        if (i >= d) continue;
        const size_t at = t * H * d + c;
        qn[at] = ld_f(U, dt, u0 + r_off + c);
        kn[at] = k[e];
        vv[at] = ld_f(U, dt, u0 + v_off + c);
        dec[at] = expf(-rate * fd_sigmoid(ld_f(Z, z_dt, t * z_stride + c) + w0[c]));
        removal[at] = fd_sigmoid(ld_f(U, dt, u0 + a_off + c) + a_bias[c]) * (k[e] * inv);
    }
}

extern "C" int illm_removal_prepare(const void* U, int dt, int u_stride, int r_off, int k_off, int v_off,
                                    int a_off, const float* a_bias, const void* Z, int z_dt, int z_stride,
                                    const float* w0, float rate, float* qn, float* kn, float* vv, float* beta,
                                    float* dec, float* removal, int T, int H, int d, void* stream) {
    if (T < 0 || H <= 0 || d <= 0 || d > 64 * FD_VEC || !illm_dtype_ok(dt) || !illm_dtype_ok(z_dt) ||
        z_stride < H * d || !fd_columns_ok(u_stride, r_off, H * d) || !fd_columns_ok(u_stride, k_off, H * d) ||
        !fd_columns_ok(u_stride, v_off, H * d) || !fd_columns_ok(u_stride, a_off, H * d) || (H + 3) / 4 > 65535)
        return ILLM_ERR_ARG;
    if (T == 0) return ILLM_OK;
    hipLaunchKernelGGL(removal_prepare_kernel, dim3(T, (H + 3) / 4), dim3(256), 0, (hipStream_t)stream, U, dt,
                       u_stride, r_off, k_off, v_off, a_off, a_bias, Z, z_dt, z_stride, w0, rate, qn, kn, vv,
                       beta, dec, removal, H, d);
    return illm_launch_status();
}

// out[t, i] = tanh(U[t, off + i]), i < n, as float32.
__global__ void __launch_bounds__(256)
tanh_columns_kernel(const void* __restrict__ U, int dt, int u_stride, int off, float* __restrict__ out, int n) {
    const size_t t = blockIdx.x;
    for (int i = threadIdx.x; i < n; i += 256) out[t * n + i] = tanhf(ld_f(U, dt, t * u_stride + off + i));
}

extern "C" int illm_tanh_columns(const void* U, int dt, int u_stride, int off, float* out, int T, int n,
                                 void* stream) {
    if (T < 0 || n <= 0 || !illm_dtype_ok(dt) || !fd_columns_ok(u_stride, off, n)) return ILLM_ERR_ARG;
    if (T == 0) return ILLM_OK;
    hipLaunchKernelGGL(tanh_columns_kernel, dim3(T), dim3(256), 0, (hipStream_t)stream, U, dt, u_stride, off, out, n);
    return illm_launch_status();
}

// ---------------------------------------------------------------- single tokens
// grid (ceil(dv / 64), H, rows); 4 waves: a lane is a column of the state, wave w holds rows [w NS, w NS +
// NS) of it (NS >= ceil(dk / 4)).  Row b belongs to the sequence in slot row_slot[b].  The head's vectors
// (k, q and, with a removal vector, the decays and the vector) are formed by the block into LDS while the
// state's rows are on their way; the waves' partial sums meet in LDS, in wave order.
#define FD_RANK_MAX 512
enum { FD_LIGHTNING = 0, FD_REMOVAL = 1, FD_RETENTION = 2, FD_TIME_MIX = 3 };
struct StepArgs {
    const float* decay;       // FD_LIGHTNING, FD_RETENTION: [H]
    const void* rates;        // FD_REMOVAL: the rates' pre-activations, rows like q's
    const float* rate_bias;   // FD_REMOVAL: [H d]
    const void* low;          // FD_REMOVAL, FD_TIME_MIX: y1 of the low-rank map, [rows, low_stride]
    int low_stride, rank;
    const void* w2;           // [H d, rank], the projections' type
    const float* w0;          // [H d]
    float rate;               // FD_REMOVAL
    const float* bonus;       // FD_TIME_MIX: [H d]
    const float* cos_sin;     // FD_RETENTION: [positions, rot / 2, 2]
    const int32_t* row_pos;
    int rot;
    float k_scale;
};

template <int NS, int DT, int MODE>
__global__ void __launch_bounds__(256)
fixed_step_kernel(const void* __restrict__ q_rows, const void* __restrict__ k_rows,
                  const void* __restrict__ v_rows, int stride, StepArgs sa, float* __restrict__ state,
                  const int32_t* __restrict__ row_slot, float* __restrict__ o, int H, int dk, int dv) {
    constexpr bool REMOVAL = MODE == FD_REMOVAL, MIX = MODE == FD_TIME_MIX, LOW = REMOVAL || MIX;
    __shared__ float sk[4 * NS], sq[4 * NS], sw[LOW ? 4 * NS : 1], sc[REMOVAL ? 4 * NS : 1];
    __shared__ float low[LOW ? FD_RANK_MAX : 1];
    __shared__ float part[LOW ? 256 : 1];
    __shared__ float red[2][4][64];
    __shared__ float redb[16];
    const int b = blockIdx.z, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, w = wave_index();
    const int col = blockIdx.x * 64 + lane, i0 = w * NS;
    const bool live = col < dv;
    const size_t u0 = (size_t)b * stride;
    float* sp = state + (((size_t)row_slot[b] * H + h) * dk) * dv + col;
    float s[NS];
#pragma unroll
    for (int ii = 0; ii < NS; ++ii) s[ii] = (live && i0 + ii < dk) ? sp[(size_t)(i0 + ii) * dv] : 0.f;
    float v = live ? ld_f(v_rows, DT, u0 + (size_t)h * dv + col) : 0.f;
    if (MODE == FD_LIGHTNING) v = fd_silu(v);
    const int i = tid;                                  // a thread a channel (dk <= 256)
    const bool mine = i < dk;
    float k = mine ? ld_f(k_rows, DT, u0 + (size_t)h * dk + i) : 0.f;
    float q = mine ? ld_f(q_rows, DT, u0 + (size_t)h * dk + i) : 0.f;
    float inv = 1.f, bonus = 0.f;
    if (LOW) {
        for (int r = tid; r < sa.rank; r += 256) low[r] = tanhf(ld_f(sa.low, DT, (size_t)b * sa.low_stride + r));
        // (the sum's barriers also publish `low`)
        if (REMOVAL) inv = 1.0f / sqrtf(block_sum(k * k, redb) + 1e-6f);
        else bonus = block_sum(mine ? q * sa.bonus[h * dk + i] * k : 0.f, redb);
        // z of the head's channels: 256 / DKP threads a channel, each a share of the rank
        constexpr int DKP = 4 * NS, SH = 256 / DKP;
        const int zi = tid % DKP, sh = tid / DKP;
        float z = 0.f;
        if (zi < dk) {
            const size_t w2 = ((size_t)h * dk + zi) * sa.rank;
            const int per = (sa.rank + SH - 1) / SH, r1 = min(sa.rank, (sh + 1) * per);
#pragma unroll 8
            for (int r = sh * per; r < r1; ++r) z = fmaf(ld_f(sa.w2, DT, w2 + r), low[r], z);
        }
        part[tid] = z;
        __syncthreads();
        if (mine) {
            z = sa.w0[h * dk + i];
#pragma unroll
            for (int x = 0; x < SH; ++x) z += part[x * DKP + i];
            if (REMOVAL) {
                sw[i] = expf(-sa.rate * fd_sigmoid(z));
                sc[i] = fd_sigmoid(ld_f(sa.rates, DT, u0 + (size_t)h * dk + i) + sa.rate_bias[h * dk + i]) * (k * inv);
            } else {
                sw[i] = expf(-expf(z));
            }
        } else if (i < DKP) {
            sw[i] = 1.f;
            if (REMOVAL) sc[i] = 0.f;
        }
    } else if (MODE == FD_RETENTION) {
        if (i < 4 * NS) { sk[i] = k; sq[i] = q; }
        __syncthreads();
        if (i < sa.rot) {
            const int half = sa.rot / 2, j = i < half ? i : i - half, other = i < half ? i + half : j;
            const float* cs = sa.cos_sin + (size_t)sa.row_pos[b] * sa.rot + 2 * j;
            const float c = cs[0], sn = i < half ? -cs[1] : cs[1];
            k = k * c + sk[other] * sn;
            q = q * c + sq[other] * sn;
        }
        k *= sa.k_scale;
        __syncthreads();
    } else {
        k = fd_silu(k); q = fd_silu(q);
    }
    if (i < 4 * NS) { sk[i] = mine ? k : 0.f; sq[i] = mine ? q : 0.f; }
    __syncthreads();
    float pa[4] = {0.f, 0.f, 0.f, 0.f};
    float read = 0.f;
    if (REMOVAL) {
#pragma unroll
        for (int ii = 0; ii < NS; ++ii) pa[ii & 3] = fmaf(s[ii], sk[i0 + ii], pa[ii & 3]);
        red[0][w][lane] = (pa[0] + pa[1]) + (pa[2] + pa[3]);
        __syncthreads();
        read = inv * ((red[0][0][lane] + red[0][1][lane]) + (red[0][2][lane] + red[0][3][lane]));
        pa[0] = pa[1] = pa[2] = pa[3] = 0.f;
    }
    const float lam = LOW ? 1.f : sa.decay[h];
#pragma unroll
    for (int ii = 0; ii < NS; ++ii) {
        if (MIX) {                                       // o from the state before the token
            pa[ii & 3] = fmaf(s[ii], sq[i0 + ii], pa[ii & 3]);
            s[ii] = fmaf(sk[i0 + ii], v, s[ii] * sw[i0 + ii]);
            continue;
        }
        if (REMOVAL) s[ii] = fmaf(-sc[i0 + ii], read, s[ii] * sw[i0 + ii]);
        else s[ii] *= lam;
        s[ii] = fmaf(sk[i0 + ii], v, s[ii]);
        pa[ii & 3] = fmaf(s[ii], sq[i0 + ii], pa[ii & 3]);
    }
    red[1][w][lane] = (pa[0] + pa[1]) + (pa[2] + pa[3]);
#pragma unroll
    for (int ii = 0; ii < NS; ++ii)
        if (live && i0 + ii < dk) sp[(size_t)(i0 + ii) * dv] = s[ii];
    __syncthreads();
    if (w == 0 && live) {
        float y = (red[1][0][lane] + red[1][1][lane]) + (red[1][2][lane] + red[1][3][lane]);
        if (MIX) y = fmaf(bonus, v, y);
        o[((size_t)b * H + h) * dv + col] = y;
    }
}

static const void* fd_at(const void* base, int dt, size_t column) {
    return (const char*)base + column * (dt == ILLM_BF16 ? 2 : 4);
}

template <int MODE>
static int fixed_step_launch(const void* q, const void* k, const void* v, int dt, int stride, StepArgs sa,
                             float* state, const int32_t* row_slot, float* o, int B, int H, int dk, int dv,
                             hipStream_t st) {
    const dim3 grid((dv + 63) / 64, H, B);
    const int ns = (dk + 3) / 4;
#define GO(NS_, DT_)                                                                                    \
    hipLaunchKernelGGL((fixed_step_kernel<NS_, DT_, MODE>), grid, dim3(256), 0, st, q, k, v, stride, sa, state, \
                       row_slot, o, H, dk, dv)
#define GO_D(NS_)                                                                                       \
    if (dt == ILLM_BF16) GO(NS_, ILLM_BF16); else GO(NS_, ILLM_F32);
    if (ns <= 4) { GO_D(4) }
    else if (ns <= 8) { GO_D(8) }
    else if (ns <= 16) { GO_D(16) }
    else if (ns <= 32) { GO_D(32) }
    else { GO_D(64) }
#undef GO_D
#undef GO
    return illm_launch_status();
}

extern "C" int illm_lightning_step(const void* U, int dt, int u_stride, int q_off, int k_off, int v_off,
                                   const float* decay, float* state, const int32_t* row_slot, float* o, int B,
                                   int H, int dk, int dv, void* stream) {
    if (B < 0 || B > 65535 || H <= 0 || H > 65535 || dk <= 0 || dk > 256 || dv <= 0 || !illm_dtype_ok(dt) ||
        !fd_columns_ok(u_stride, q_off, H * dk) || !fd_columns_ok(u_stride, k_off, H * dk) ||
        !fd_columns_ok(u_stride, v_off, H * dv))
        return ILLM_ERR_ARG;
    if (B == 0) return ILLM_OK;
    StepArgs sa = {};
    sa.decay = decay;
    return fixed_step_launch<FD_LIGHTNING>(fd_at(U, dt, q_off), fd_at(U, dt, k_off), fd_at(U, dt, v_off), dt, u_stride,
                                           sa, state, row_slot, o, B, H, dk, dv, (hipStream_t)stream);
}

extern "C" int illm_removal_step(const void* U, int dt, int u_stride, int r_off, int k_off, int v_off, int a_off,
                                 const float* a_bias, int w1_off, int rank, const void* w2, const float* w0,
                                 float rate, float* state, const int32_t* row_slot, float* o, int B, int H,
                                 int d, void* stream) {
    if (B < 0 || B > 65535 || H <= 0 || H > 65535 || d <= 0 || d > 256 || rank <= 0 || rank > FD_RANK_MAX ||
        !illm_dtype_ok(dt) || !fd_columns_ok(u_stride, r_off, H * d) || !fd_columns_ok(u_stride, k_off, H * d) ||
        !fd_columns_ok(u_stride, v_off, H * d) || !fd_columns_ok(u_stride, a_off, H * d) ||
        !fd_columns_ok(u_stride, w1_off, rank))
        return ILLM_ERR_ARG;
    if (B == 0) return ILLM_OK;
    StepArgs sa = {};
    sa.rates = fd_at(U, dt, a_off); sa.rate_bias = a_bias; sa.rate = rate;
    sa.low = fd_at(U, dt, w1_off); sa.low_stride = u_stride; sa.rank = rank; sa.w2 = w2; sa.w0 = w0;
    return fixed_step_launch<FD_REMOVAL>(fd_at(U, dt, r_off), fd_at(U, dt, k_off), fd_at(U, dt, v_off), dt, u_stride,
                                         sa, state, row_slot, o, B, H, d, d, (hipStream_t)stream);
}

extern "C" int illm_retention_step(const void* U, int dt, int u_stride, int q_off, int k_off, int v_off,
                                   const float* decay, const float* cos_sin, int n_positions, int rot, float k_scale,
                                   const int32_t* row_pos, float* state, const int32_t* row_slot, float* o, int B,
                                   int H, int dk, int dv, void* stream) {
    if (B < 0 || B > 65535 || H <= 0 || H > 65535 || dk <= 0 || dk > 256 || dv <= 0 || !illm_dtype_ok(dt) ||
        rot < 0 || rot % 2 || rot > dk || (rot > 0 && (!cos_sin || n_positions <= 0 || !row_pos)) ||
        !fd_columns_ok(u_stride, q_off, H * dk) || !fd_columns_ok(u_stride, k_off, H * dk) ||
        !fd_columns_ok(u_stride, v_off, H * dv))
        return ILLM_ERR_ARG;
    if (B == 0) return ILLM_OK;
    StepArgs sa = {};
    sa.decay = decay; sa.cos_sin = cos_sin; sa.row_pos = row_pos; sa.rot = rot; sa.k_scale = k_scale;
    return fixed_step_launch<FD_RETENTION>(fd_at(U, dt, q_off), fd_at(U, dt, k_off), fd_at(U, dt, v_off), dt, u_stride,
                                           sa, state, row_slot, o, B, H, dk, dv, (hipStream_t)stream);
}

extern "C" int illm_time_mix_step(const void* r, const void* k, const void* v, int dt, int stride, const void* low,
                                  int low_stride, int rank, const void* w2, const float* w0, const float* bonus,
                                  float* state, const int32_t* row_slot, float* o, int B, int H, int d, void* stream) {
    if (B < 0 || B > 65535 || H <= 0 || H > 65535 || d <= 0 || d > 256 || rank <= 0 || rank > FD_RANK_MAX ||
        !illm_dtype_ok(dt) || stride < H * d || low_stride < rank)
        return ILLM_ERR_ARG;
    if (B == 0) return ILLM_OK;
    StepArgs sa = {};
    sa.low = low; sa.low_stride = low_stride; sa.rank = rank; sa.w2 = w2; sa.w0 = w0; sa.bonus = bonus;
    return fixed_step_launch<FD_TIME_MIX>(r, k, v, dt, stride, sa, state, row_slot, o, B, H, d, d,
                                          (hipStream_t)stream);
}

// ---------------------------------------------------------------- lightning attention in chunks
// A step's rows of a sequence in chunks of FD_CHUNK tokens (the last one shorter, n_c tokens):
//   chunk_sums    per (chunk, head): sum_i lam^(n_c - 1 - i) k_i v_i^T, the chunk's part of the state
//   chunk_carry   per head, chunk after chunk: the state at every chunk's start (in place of the sums)
//                 and the sequence's last state back into the slot
//   chunk_rows    per (chunk, head): o_i = lam^(i + 1) S_start^T q_i + sum_(j <= i) lam^(i - j) (q_i . k_j) v_j
// Products on the matrix cores' float32 instruction (32x32x2: float32 operands, products and sums).
// Chunk c of sequence b lies at place cu[b] / FD_CHUNK + b + c of `part` [places][H][dk][dv].  Key and value
// sizes up to 128 in steps of 4, filled up with zeros to whole tiles of 32 (KT, VT).
#define FD_CHUNK 64
typedef float fd_f32x16_t __attribute__((ext_vector_type(16)));

template <int DT, bool SILU>
__device__ __forceinline__ float4 ld4_act(const void* p, size_t at) {
    float4 x = ld_f4(p, DT, at / 4);
    if (!SILU) return x;
    x.x = fd_silu(x.x); x.y = fd_silu(x.y); x.z = fd_silu(x.z); x.w = fd_silu(x.w);
    return x;
}

// grid (chunks, H, sequences); 256 threads.  Both operands lie in LDS as [token][channel]; a wave takes
// every fourth tile of 32 x 32 of the sum.
template <int KDT, int DT, bool SILU, int KT, int VT>
__global__ void __launch_bounds__(256)
lightning_chunk_sums_kernel(const void* __restrict__ K, int k_stride, const void* __restrict__ V, int v_stride,
                            const float* __restrict__ decay, float* __restrict__ part,
                            const int32_t* __restrict__ cu, int H, int dk, int dv) {
    constexpr int DKP = 32 * KT, DVP = 32 * VT, NT = (KT * VT + 3) / 4;
    __shared__ float ks[FD_CHUNK * DKP];
    __shared__ float vs[FD_CHUNK * DVP];
    __shared__ float pw[FD_CHUNK];
    const int b = blockIdx.z, h = blockIdx.y, c = blockIdx.x, tid = threadIdx.x;
    const int r0 = cu[b], n = cu[b + 1] - r0, t0 = c * FD_CHUNK;
    if (t0 >= n) return;                                // the whole block
    const int nc = min(FD_CHUNK, n - t0);
    if (tid < FD_CHUNK) pw[tid] = tid < nc ? powf(decay[h], (float)(nc - 1 - tid)) : 0.f;
    __syncthreads();
    for (int e = tid; e < FD_CHUNK * (DKP / 4); e += 256) {
        const int row = e / (DKP / 4), d = 4 * (e % (DKP / 4));
        float4 x = make_float4(0.f, 0.f, 0.f, 0.f);
        if (row < nc && d < dk) x = ld4_act<KDT, SILU>(K, (size_t)(r0 + t0 + row) * k_stride + (size_t)h * dk + d);
        const float f = pw[row];
        *(float4*)(ks + row * DKP + d) = make_float4(x.x * f, x.y * f, x.z * f, x.w * f);
    }
    for (int e = tid; e < FD_CHUNK * (DVP / 4); e += 256) {
        const int row = e / (DVP / 4), d = 4 * (e % (DVP / 4));
        float4 x = make_float4(0.f, 0.f, 0.f, 0.f);
        if (row < nc && d < dv) x = ld4_act<DT, SILU>(V, (size_t)(r0 + t0 + row) * v_stride + (size_t)h * dv + d);
        *(float4*)(vs + row * DVP + d) = x;
    }
    __syncthreads();
    const int lane = tid & 63, w = wave_index(), col = lane & 31, half = lane >> 5;
    float* dst = part + (((size_t)(r0 / FD_CHUNK + b + c)) * H + h) * dk * dv;
#pragma unroll
    for (int x = 0; x < NT; ++x) {
        const int tile = w + 4 * x;
        if (tile >= KT * VT) continue;
        const int m0 = 32 * (tile / VT), n0 = 32 * (tile % VT);
        fd_f32x16_t acc;
#pragma unroll
        for (int v = 0; v < 16; ++v) acc[v] = 0.f;
#pragma unroll 8
        for (int s2 = 0; s2 < FD_CHUNK / 2; ++s2)
            acc = __builtin_amdgcn_mfma_f32_32x32x2f32(ks[(2 * s2 + half) * DKP + m0 + col],
                                                       vs[(2 * s2 + half) * DVP + n0 + col], acc, 0, 0, 0);
#pragma unroll
        for (int v = 0; v < 16; ++v) {
            const int m = m0 + 8 * (v >> 2) + 4 * half + (v & 3), nn = n0 + col;
            if (m < dk && nn < dv) dst[(size_t)m * dv + nn] = acc[v];
        }
    }
}

// grid (ceil(dk dv / 1024), H, sequences); 256 threads, 4 neighbouring numbers each (dv % 4 == 0).
#define FD_AHEAD 8
__global__ void __launch_bounds__(256)
lightning_chunk_carry_kernel(float* __restrict__ part, const float* __restrict__ decay,
                             float* __restrict__ state, const int32_t* __restrict__ cu,
                             const int32_t* __restrict__ seq_slot, int H, int dk, int dv) {
    const int b = blockIdx.z, h = blockIdx.y, i4 = blockIdx.x * 256 + threadIdx.x;
    const int r0 = cu[b], n = cu[b + 1] - r0, n4 = dk * dv / 4;
    if (n <= 0 || i4 >= n4) return;
    const int chunks = (n + FD_CHUNK - 1) / FD_CHUNK;
    const float lam = decay[h];
    const float full = powf(lam, (float)FD_CHUNK), last = powf(lam, (float)(n - (chunks - 1) * FD_CHUNK));
    float4* sp = (float4*)(state + ((size_t)seq_slot[b] * H + h) * dk * dv) + i4;
    float4* pp = (float4*)(part + ((size_t)(r0 / FD_CHUNK + b) * H + h) * dk * dv) + i4;
    const size_t step = (size_t)H * n4;
    float4 S = *sp;
    for (int c0 = 0; c0 < chunks; c0 += FD_AHEAD) {
        float4 add[FD_AHEAD];
#pragma unroll
        for (int x = 0; x < FD_AHEAD; ++x)
            if (c0 + x < chunks) add[x] = pp[(size_t)(c0 + x) * step];
#pragma unroll
        for (int x = 0; x < FD_AHEAD; ++x) {
            if (c0 + x >= chunks) continue;
            pp[(size_t)(c0 + x) * step] = S;
            const float f = c0 + x == chunks - 1 ? last : full;
            S.x = fmaf(f, S.x, add[x].x); S.y = fmaf(f, S.y, add[x].y);
            S.z = fmaf(f, S.z, add[x].z); S.w = fmaf(f, S.w, add[x].w);
        }
    }
    *sp = S;
}

// grid (chunks, H, sequences); 256 threads: wave w takes the chunk's 32 tokens of tile w % 2 and every
// second value tile from w / 2 on.  Both products are kept transposed, so that a lane's column is its
// token: scores^T = K . Q^T leaves the 16 scores of token (lane % 32) in a lane and its partner 32 lanes
// on, and in o^T = V^T . P^T they are the second operand as they stand.  k and v lie in LDS, q in
// registers; the start state is read straight from memory (32 neighbouring values a row).
template <int KDT, int DT, bool SILU, int KT, int VT>
__global__ void __launch_bounds__(256, 2)
lightning_chunk_rows_kernel(const void* __restrict__ Q, const void* __restrict__ K, int k_stride,
                            const void* __restrict__ V, int v_stride,
                            const float* __restrict__ decay, const float* __restrict__ part,
                            const int32_t* __restrict__ cu, float* __restrict__ o, int H, int dk, int dv) {
    constexpr int DKP = 32 * KT, DVP = 32 * VT, KLD = DKP + 1, VW = (VT + 1) / 2;
    __shared__ float ks[FD_CHUNK * KLD];
    __shared__ float vs[FD_CHUNK * DVP];
    __shared__ float pw[FD_CHUNK + 1];
    const int b = blockIdx.z, h = blockIdx.y, c = blockIdx.x, tid = threadIdx.x;
    const int r0 = cu[b], n = cu[b + 1] - r0, t0 = c * FD_CHUNK;
    if (t0 >= n) return;                                // the whole block
    const int nc = min(FD_CHUNK, n - t0);
    const int lane = tid & 63, w = wave_index(), col = lane & 31, half = lane >> 5;
    const int it = w & 1, i = 32 * it + col;            // the lane's token within the chunk
    if (tid <= FD_CHUNK) pw[tid] = powf(decay[h], (float)tid);
    float qr[DKP / 2];                                  // dims 2 s + half (zeros beyond dk)
    {
        const size_t at = (size_t)(r0 + t0 + min(i, nc - 1)) * k_stride + (size_t)h * dk;
#pragma unroll
        for (int j = 0; j < DKP / 4; ++j) {
            float4 x = make_float4(0.f, 0.f, 0.f, 0.f);
            if (4 * j < dk) x = ld4_act<KDT, SILU>(Q, at + 4 * j);
            qr[2 * j] = half ? x.y : x.x;
            qr[2 * j + 1] = half ? x.w : x.z;
        }
    }
    for (int e = tid; e < FD_CHUNK * (DKP / 4); e += 256) {
        const int row = e / (DKP / 4), d = 4 * (e % (DKP / 4));
        float4 x = make_float4(0.f, 0.f, 0.f, 0.f);
        if (row < nc && d < dk) x = ld4_act<KDT, SILU>(K, (size_t)(r0 + t0 + row) * k_stride + (size_t)h * dk + d);
        float* to = ks + row * KLD + d;
        to[0] = x.x; to[1] = x.y; to[2] = x.z; to[3] = x.w;
    }
    for (int e = tid; e < FD_CHUNK * (DVP / 4); e += 256) {
        const int row = e / (DVP / 4), d = 4 * (e % (DVP / 4));
        float4 x = make_float4(0.f, 0.f, 0.f, 0.f);
        if (row < nc && d < dv) x = ld4_act<DT, SILU>(V, (size_t)(r0 + t0 + row) * v_stride + (size_t)h * dv + d);
        *(float4*)(vs + row * DVP + d) = x;
    }
    __syncthreads();
    if (32 * it >= nc) return;                          // (no barrier follows)
    const float* S = part + (((size_t)(r0 / FD_CHUNK + b + c)) * H + h) * dk * dv;
    fd_f32x16_t acc[VW];
#pragma unroll
    for (int t = 0; t < VW; ++t) {
        const int n0 = 32 * (2 * t + (w >> 1));
#pragma unroll
        for (int v = 0; v < 16; ++v) acc[t][v] = 0.f;
        if (n0 >= dv) continue;
        // (rows beyond dk meet zeros of q and columns beyond dv are not stored: read a valid place, no branch)
        const float* Sc = S + min(n0 + col, dv - 1);
#pragma unroll
        for (int s0 = 0; s0 < DKP / 2; s0 += 16) {
            float a[16];
#pragma unroll
            for (int x = 0; x < 16; ++x) a[x] = Sc[(size_t)min(2 * (s0 + x) + half, dk - 1) * dv];
#pragma unroll
            for (int x = 0; x < 16; ++x)
                acc[t] = __builtin_amdgcn_mfma_f32_32x32x2f32(a[x], qr[s0 + x], acc[t], 0, 0, 0);
        }
    }
    const float f = pw[min(i, nc - 1) + 1];
#pragma unroll
    for (int t = 0; t < VW; ++t)
#pragma unroll
        for (int v = 0; v < 16; ++v) acc[t][v] *= f;
    for (int jt = 0; jt <= it; ++jt) {
        fd_f32x16_t sc;
#pragma unroll
        for (int v = 0; v < 16; ++v) sc[v] = 0.f;
        const float* kr = ks + (32 * jt + col) * KLD + half;
#pragma unroll
        for (int s2 = 0; s2 < DKP / 2; ++s2)
            sc = __builtin_amdgcn_mfma_f32_32x32x2f32(kr[2 * s2], qr[s2], sc, 0, 0, 0);
#pragma unroll
        for (int v = 0; v < 16; ++v) {
            const int j = 32 * jt + 8 * (v >> 2) + 4 * half + (v & 3);
            sc[v] = j <= i ? sc[v] * pw[i - j] : 0.f;
        }
#pragma unroll
        for (int t = 0; t < VW; ++t) {
            const int n0 = 32 * (2 * t + (w >> 1));
            if (n0 >= DVP) continue;
            const float* vr = vs + (32 * jt + 4 * half) * DVP + n0 + col;
#pragma unroll
            for (int v = 0; v < 16; ++v)
                acc[t] = __builtin_amdgcn_mfma_f32_32x32x2f32(vr[(8 * (v >> 2) + (v & 3)) * DVP], sc[v], acc[t], 0, 0, 0);
        }
    }
    if (i >= nc) return;
    float* op = o + ((size_t)(r0 + t0 + i) * H + h) * dv;
#pragma unroll
    for (int t = 0; t < VW; ++t)
#pragma unroll
        for (int g = 0; g < 4; ++g) {
            const int d = 32 * (2 * t + (w >> 1)) + 8 * g + 4 * half;
            if (d < dv)
                *(float4*)(op + d) = make_float4(acc[t][4 * g], acc[t][4 * g + 1], acc[t][4 * g + 2], acc[t][4 * g + 3]);
        }
}

extern "C" int illm_lightning_chunk(void) { return FD_CHUNK; }

// q and k rows of type KDT and k_stride numbers, v rows of type DT and v_stride.
template <int KDT, int DT, bool SILU>
static int chunks_launch(const void* Q, const void* K, int k_stride, const void* V, int v_stride, const float* decay,
                         float* state, float* part, const int32_t* cu, const int32_t* seq_slot, float* o,
                         int n_seqs, int max_rows, int H, int dk, int dv, hipStream_t st) {
    const dim3 grid((max_rows + FD_CHUNK - 1) / FD_CHUNK, H, n_seqs);
    const int kt = (dk + 31) / 32, vt = (dv + 31) / 32;
#define GO(KT_, VT_)                                                                                    \
    do {                                                                                                \
        hipLaunchKernelGGL((lightning_chunk_sums_kernel<KDT, DT, SILU, KT_, VT_>), grid, dim3(256), 0, st, K, \
                           k_stride, V, v_stride, decay, part, cu, H, dk, dv);                          \
        hipLaunchKernelGGL(lightning_chunk_carry_kernel, dim3((dk * dv / 4 + 255) / 256, H, n_seqs), dim3(256), 0, \
                           st, part, decay, state, cu, seq_slot, H, dk, dv);                            \
        hipLaunchKernelGGL((lightning_chunk_rows_kernel<KDT, DT, SILU, KT_, VT_>), grid, dim3(256), 0, st, Q, K, \
                           k_stride, V, v_stride, decay, part, cu, o, H, dk, dv);                       \
    } while (0)
#define GO_V(KT_)                                                                                       \
    switch (vt) { case 1: GO(KT_, 1); break; case 2: GO(KT_, 2); break;                                 \
                  case 3: GO(KT_, 3); break; default: GO(KT_, 4); break; }
    switch (kt) { case 1: GO_V(1) break; case 2: GO_V(2) break; case 3: GO_V(3) break; default: GO_V(4) break; }
#undef GO_V
#undef GO
    return illm_launch_status();
}

static bool chunks_sizes_ok(int n_seqs, int max_rows, int H, int dk, int dv) {
    return n_seqs >= 0 && n_seqs <= 65535 && max_rows >= 0 && H > 0 && H <= 65535 && dk > 0 && dk <= 128 &&
           dk % 4 == 0 && dv > 0 && dv <= 128 && dv % 4 == 0;
}

// `part`: (T / FD_CHUNK + n_seqs + 1) H dk dv floats.
extern "C" int illm_lightning_chunks(const void* U, int dt, int u_stride, int q_off, int k_off, int v_off,
                                     const float* decay, float* state, float* part, const int32_t* cu,
                                     const int32_t* seq_slot, float* o, int n_seqs, int max_rows, int H, int dk,
                                     int dv, void* stream) {
    if (!chunks_sizes_ok(n_seqs, max_rows, H, dk, dv) || !illm_dtype_ok(dt) || u_stride % 4 || q_off % 4 ||
        k_off % 4 || v_off % 4 || !fd_columns_ok(u_stride, q_off, H * dk) || !fd_columns_ok(u_stride, k_off, H * dk) ||
        !fd_columns_ok(u_stride, v_off, H * dv) || !part)
        return ILLM_ERR_ARG;
    if (n_seqs == 0 || max_rows == 0) return ILLM_OK;
    const void *q = fd_at(U, dt, q_off), *k = fd_at(U, dt, k_off), *v = fd_at(U, dt, v_off);
    if (dt == ILLM_BF16)
        return chunks_launch<ILLM_BF16, ILLM_BF16, true>(q, k, u_stride, v, u_stride, decay, state, part, cu, seq_slot,
                                                         o, n_seqs, max_rows, H, dk, dv, (hipStream_t)stream);
    return chunks_launch<ILLM_F32, ILLM_F32, true>(q, k, u_stride, v, u_stride, decay, state, part, cu, seq_slot, o,
                                                   n_seqs, max_rows, H, dk, dv, (hipStream_t)stream);
}

// The same chunks without activations: qn, kn float32 [T, H, dk] (illm_retention_prepare), v in U's columns
// v_off .. as stored.
extern "C" int illm_retention_chunks(const float* qn, const float* kn, const void* U, int dt, int u_stride, int v_off,
                                     const float* decay, float* state, float* part, const int32_t* cu,
                                     const int32_t* seq_slot, float* o, int n_seqs, int max_rows, int H, int dk,
                                     int dv, void* stream) {
    if (!chunks_sizes_ok(n_seqs, max_rows, H, dk, dv) || !illm_dtype_ok(dt) || u_stride % 4 || v_off % 4 ||
        !fd_columns_ok(u_stride, v_off, H * dv) || !part)
        return ILLM_ERR_ARG;
    if (n_seqs == 0 || max_rows == 0) return ILLM_OK;
    const void* v = fd_at(U, dt, v_off);
    if (dt == ILLM_BF16)
        return chunks_launch<ILLM_F32, ILLM_BF16, false>(qn, kn, H * dk, v, u_stride, decay, state, part, cu, seq_slot,
                                                         o, n_seqs, max_rows, H, dk, dv, (hipStream_t)stream);
    return chunks_launch<ILLM_F32, ILLM_F32, false>(qn, kn, H * dk, v, u_stride, decay, state, part, cu, seq_slot, o,
                                                    n_seqs, max_rows, H, dk, dv, (hipStream_t)stream);
}

// ---------------------------------------------------------------- behind the recurrence
// out[r, j] = o[r, j] / sqrt(mean over j's part of o^2 + eps) * w[j] * act(Z[r, z_off + j]) with the row of
// `width` numbers in `groups` equal parts (w null: no weight); act = silu (gate_kind 0) or sigmoid (1).
// Parts of up to 512 numbers: grid (rows, ceil(groups / 4)), a wave a part; longer ones: grid (rows,
// groups), a block a part.
__device__ __forceinline__ float fd_gate(float z, int gate_kind) { return gate_kind ? fd_sigmoid(z) : fd_silu(z); }

template <bool WAVE>
__global__ void __launch_bounds__(256)
group_norm_gate_kernel(const float* __restrict__ o, const void* __restrict__ w, int w_dt,
                       const void* __restrict__ Z, int z_dt, int z_stride, int z_off, int gate_kind,
                       void* __restrict__ out, int out_dt, int width, int part, float eps) {
    __shared__ float red[16];
    const size_t r = blockIdx.x;
    const int g = WAVE ? blockIdx.y * 4 + wave_index() : blockIdx.y;
    const int j0 = g * part, t = WAVE ? threadIdx.x & 63 : threadIdx.x, step = WAVE ? 64 : 256;
    if (WAVE && j0 >= width) return;
    const float* op = o + r * width + j0;
    float ss = 0.f;
    if (part % 4 == 0 && z_stride % 4 == 0 && z_off % 4 == 0) {
        for (int j = t; j < part / 4; j += step) {
            const float4 x = ((const float4*)op)[j];
            ss += x.x * x.x + x.y * x.y + x.z * x.z + x.w * x.w;
        }
        ss = WAVE ? wave_sum(ss) : block_sum(ss, red);
        const float inv = 1.0f / sqrtf(ss / (float)part + eps);
        for (int j = t; j < part / 4; j += step) {
            float4 x = ((const float4*)op)[j];
            const float4 ww = w ? ld_f4(w, w_dt, j0 / 4 + j) : make_float4(1.f, 1.f, 1.f, 1.f), z = ld_f4(Z, z_dt, (r * z_stride + z_off + j0) / 4 + j);
            x.x = (x.x * inv) * ww.x * fd_gate(z.x, gate_kind);
            x.y = (x.y * inv) * ww.y * fd_gate(z.y, gate_kind);
            x.z = (x.z * inv) * ww.z * fd_gate(z.z, gate_kind);
            x.w = (x.w * inv) * ww.w * fd_gate(z.w, gate_kind);
            st_f4(out, out_dt, (r * width + j0) / 4 + j, x);
        }
        return;
    }
    for (int j = t; j < part; j += step) ss = fmaf(op[j], op[j], ss);
    ss = WAVE ? wave_sum(ss) : block_sum(ss, red);
    const float inv = 1.0f / sqrtf(ss / (float)part + eps);
    for (int j = t; j < part; j += step)
        st_f(out, out_dt, r * width + j0 + j, (op[j] * inv) * (w ? ld_f(w, w_dt, j0 + j) : 1.f) *
                                                  fd_gate(ld_f(Z, z_dt, r * z_stride + z_off + j0 + j), gate_kind));
}

extern "C" int illm_group_norm_gate(const float* o, const void* w, int w_dt, const void* Z, int z_dt, int z_stride,
                                    int z_off, int gate_kind, void* out, int out_dt, int T, int width, int groups,
                                    float eps, void* stream) {
    if (T < 0 || width <= 0 || groups <= 0 || groups > 65535 || width % groups || (w && !illm_dtype_ok(w_dt)) ||
        !illm_dtype_ok(z_dt) || !illm_dtype_ok(out_dt) || !fd_columns_ok(z_stride, z_off, width) ||
        (gate_kind != 0 && gate_kind != 1))
        return ILLM_ERR_ARG;
    if (T == 0) return ILLM_OK;
    const int part = width / groups;
    if (part <= 512)
        hipLaunchKernelGGL(group_norm_gate_kernel<true>, dim3(T, (groups + 3) / 4), dim3(256), 0, (hipStream_t)stream,
                           o, w, w_dt, Z, z_dt, z_stride, z_off, gate_kind, out, out_dt, width, part, eps);
    else
        hipLaunchKernelGGL(group_norm_gate_kernel<false>, dim3(T, groups), dim3(256), 0, (hipStream_t)stream, o, w,
                           w_dt, Z, z_dt, z_stride, z_off, gate_kind, out, out_dt, width, part, eps);
    return illm_launch_status();
}
