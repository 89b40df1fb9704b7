// streams.hip — a residual stream kept as SEVERAL parallel streams (hyper-connections).  In front of a sublayer the streams are weighted into the one row it reads; behind
// it every stream becomes a mixture of all old ones plus a share of the sublayer's output:
//   u = sum_n in[n] x_n;  y = sublayer(rms_norm(u) w);  x_t <- sum_n mix[n, t] x_n + mult out[t] y   (all t at once, from the old x)
// k_stream_step is what lies between two sublayers, in one launch: the update with one sublayer's (mix, out), then the weighting and the norm in front of the next.
// Memory of the result: the normed rows [E, T] first (contiguous: the operand of the next mat-muls), then the streams as N planes [E, T].
// Everything is f32; the norm's sum of squares is f64 as in the other norm kernels.
//
// One workgroup per token row.  A thread owns groups of four neighbouring entries of the row: it reads the N old streams and y there, keeps the N new values' weighted sum in
// registers until the row's sum of squares is known, and reads nothing twice.  Rows that are no multiple of four entries go entry by entry.
#include <algorithm>

#include "dev_util.h"
#include "kernels.h"

namespace mi355x {

constexpr int STREAM_R = 8;  // groups of four entries a thread may own: rows of up to 4 * 1024 * 8 entries

__device__ __forceinline__ double stream_block_sum(double v, double * sh) {
    for (int o = 32; o > 0; o >>= 1) v += __shfl_xor(v, o, 64);
    if ((threadIdx.x & 63) == 0) sh[threadIdx.x >> 6] = v;
    __syncthreads();
    double t = 0.0;
    for (int i = 0; i < (int) (blockDim.x >> 6); ++i) t += sh[i];
    return t;
}

// the new value of stream t at one entry, from the old values x[0 .. N) and the sublayer's y (no old streams: every stream starts as y)
template <int N> __device__ __forceinline__ float stream_next(const bool have_x, const float (&x)[N], const float y, const float (&m)[N][N], const float (&o)[N], const int t) {
    if (!have_x) return y;
    float v = m[0][t] * x[0];
#pragma unroll
    for (int n = 1; n < N; ++n) v = fmaf(m[n][t], x[n], v);
    return fmaf(o[t], y, v);
}

template <int N, bool VEC>
__global__ void __launch_bounds__(1024) k_stream_step(const stream_step_args A) {
    __shared__ double sh[16];
    const int64_t E = A.E, r = blockIdx.x, src = A.ids ? A.ids[r] : r;
    const bool have_x = A.x != nullptr, keep_x = A.x_out != nullptr;
    const float * __restrict__ y = A.y + src * E;
    const float * __restrict__ x = have_x ? A.x + src * E : nullptr;
    float * __restrict__ h = A.h + r * E;
    float m[N][N], o[N], a[N];
#pragma unroll
    for (int n = 0; n < N; ++n) {
        a[n] = A.in ? A.in[n] : 1.0f;
        o[n] = have_x ? A.mult * A.out[n] : 0.0f;
#pragma unroll
        for (int t = 0; t < N; ++t) m[n][t] = have_x ? A.mix[n * N + t] : 0.0f;
    }
    double ss = 0.0;
    if constexpr (VEC) {
        const int64_t n4 = E >> 2;
        float4 u[STREAM_R];
#pragma unroll
        for (int k = 0; k < STREAM_R; ++k) {
            const int64_t i = threadIdx.x + (int64_t) k * blockDim.x;
            if (i < n4) {
                const float4 yv = ((const float4 *) y)[i];
                float4 xv[N];
#pragma unroll
                for (int n = 0; n < N; ++n) xv[n] = have_x ? ((const float4 *) (x + n * A.x_plane))[i] : make_float4(0.f, 0.f, 0.f, 0.f);
                float x0[N], x1[N], x2[N], x3[N];
#pragma unroll
                for (int n = 0; n < N; ++n) { x0[n] = xv[n].x; x1[n] = xv[n].y; x2[n] = xv[n].z; x3[n] = xv[n].w; }
                float4 acc = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
                for (int t = 0; t < N; ++t) {
                    float4 v;
                    v.x = stream_next<N>(have_x, x0, yv.x, m, o, t);
                    v.y = stream_next<N>(have_x, x1, yv.y, m, o, t);
                    v.z = stream_next<N>(have_x, x2, yv.z, m, o, t);
                    v.w = stream_next<N>(have_x, x3, yv.w, m, o, t);
                    if (keep_x) ((float4 *) (A.x_out + t * A.xo_plane + r * E))[i] = v;
                    acc.x = fmaf(a[t], v.x, acc.x); acc.y = fmaf(a[t], v.y, acc.y); acc.z = fmaf(a[t], v.z, acc.z); acc.w = fmaf(a[t], v.w, acc.w);
                }
                u[k] = acc;
                ss += (double) (acc.x * acc.x) + (double) (acc.y * acc.y) + (double) (acc.z * acc.z) + (double) (acc.w * acc.w);
            }
        }
        ss = stream_block_sum(ss, sh);
        const float scale = 1.0f / sqrtf((float) (ss / (double) E) + A.eps);
#pragma unroll
        for (int k = 0; k < STREAM_R; ++k) {
            const int64_t i = threadIdx.x + (int64_t) k * blockDim.x;
            if (i < n4) {
                const float4 w = ((const float4 *) A.w)[i];
                ((float4 *) h)[i] = make_float4(u[k].x * scale * w.x, u[k].y * scale * w.y, u[k].z * scale * w.z, u[k].w * scale * w.w);
            }
        }
    } else {
        for (int64_t i = threadIdx.x; i < E; i += blockDim.x) {
            float xv[N], acc = 0.0f;
#pragma unroll
            for (int n = 0; n < N; ++n) xv[n] = have_x ? x[n * A.x_plane + i] : 0.0f;
            const float yv = y[i];
#pragma unroll
            for (int t = 0; t < N; ++t) {
                const float v = stream_next<N>(have_x, xv, yv, m, o, t);
                if (keep_x) A.x_out[t * A.xo_plane + r * E + i] = v;
                acc = fmaf(a[t], v, acc);
            }
            h[i] = acc;
            ss += (double) (acc * acc);
        }
        ss = stream_block_sum(ss, sh);
        const float scale = 1.0f / sqrtf((float) (ss / (double) E) + A.eps);
        for (int64_t i = threadIdx.x; i < E; i += blockDim.x) h[i] = h[i] * scale * A.w[i];  // (a thread re-reads only what it wrote)
    }
}

void launch_stream_step(hipStream_t s, const stream_step_args & a, int n_streams, int64_t rows) {
    if (rows == 0 || a.E == 0) return;
    const uintptr_t at = (uintptr_t) a.y | (uintptr_t) a.x | (uintptr_t) a.h | (uintptr_t) a.x_out | (uintptr_t) a.w | (uintptr_t) (a.x_plane * 4) | (uintptr_t) (a.xo_plane * 4);
    const bool vec = (a.E & 3) == 0 && (at & 15) == 0 && a.E <= (int64_t) 4 * 1024 * STREAM_R;
    const int64_t units = vec ? a.E / 4 : a.E;
    // a prompt portion has a workgroup per token: 256 threads with up to two groups each; a decode step's few rows are spread over as many threads as they have groups
    const int64_t most = rows >= 256 ? std::max<int64_t>(256, (units + 1) / 2) : 1024;
    int nt = (int) std::min<int64_t>(1024, (std::min(units, most) + 63) / 64 * 64);
    if (vec) nt = (int) std::max<int64_t>(nt, std::min<int64_t>(1024, ((units + STREAM_R - 1) / STREAM_R + 63) / 64 * 64));
#define MI_STREAM(NS) case NS: if (vec) hipLaunchKernelGGL((k_stream_step<NS, true>), dim3((unsigned) rows), dim3(nt), 0, s, a); \
                               else hipLaunchKernelGGL((k_stream_step<NS, false>), dim3((unsigned) rows), dim3(nt), 0, s, a); break;
    switch (n_streams) {
        MI_STREAM(1) MI_STREAM(2) MI_STREAM(3) MI_STREAM(4) MI_STREAM(5) MI_STREAM(6) MI_STREAM(7) MI_STREAM(8)
        default: break;
    }
#undef MI_STREAM
}

MI_TU_TOUCH(streams)

}  // namespace mi355x
