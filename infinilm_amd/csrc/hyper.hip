// A residual stream kept in several copies that the sublayers read and write through small weights ("hyper-connections").
//
//   ilm_hyper_update    rows X [T, n, H] float.  With a branch y (rows, or float parts of a K-split product that are summed
//       first) a token's streams are first made anew, X' = M^T X + outer(b, alpha y) (M[s, t]: from stream s to t); then the next
//       sublayer's input is read, u = a X' (a absent: the plain sum), and normed:
//       x = u / sqrt(mean(u^2) + eps) * (w + w_offset); without w, x is u itself.  `base` [T, H]: every old stream is this one
//       row (the start, before any branch has made the streams differ).  X' is written to X if asked for.
//
// A block a row: a thread holds its elements of all streams at once, so every stream is read once and written once, and the
// row read stays in LDS between its sum of squares and the result.  Everything is float; sums run in an order that depends
// on the sizes alone.
#include "common.h"

#define HY_MAX_STREAMS 16
#define HY_MAX_H 16384
#define HY_PB 4        // parts of a branch whose loads are in flight together

template <int VEC>
__device__ __forceinline__ void hy_load(const void* p, size_t i, int dt, float (&v)[VEC]) {
    if constexpr (VEC == 4) {
        if (dt == ILM_DTYPE_F32) {
            const float4 t = *reinterpret_cast<const float4*>((const float*)p + i);
            v[0] = t.x; v[1] = t.y; v[2] = t.z; v[3] = t.w;
        } else {
            const uint2 t = *reinterpret_cast<const uint2*>((const uint16_t*)p + i);
            v[0] = __uint_as_float(t.x << 16); v[1] = __uint_as_float(t.x & 0xffff0000u);
            v[2] = __uint_as_float(t.y << 16); v[3] = __uint_as_float(t.y & 0xffff0000u);
        }
    } else {
        v[0] = dt == ILM_DTYPE_F32 ? ((const float*)p)[i] : bf16_bits_to_f32(((const uint16_t*)p)[i]);
    }
}

template <int VEC>
__device__ __forceinline__ void hy_store(void* p, size_t i, int dt, const float (&v)[VEC]) {
    if constexpr (VEC == 4) {
        if (dt == ILM_DTYPE_F32) {
            *reinterpret_cast<float4*>((float*)p + i) = make_float4(v[0], v[1], v[2], v[3]);
        } else {
            uint2 o;
            o.x = (uint32_t)from_f32<bf16>(v[0]).bits | ((uint32_t)from_f32<bf16>(v[1]).bits << 16);
            o.y = (uint32_t)from_f32<bf16>(v[2]).bits | ((uint32_t)from_f32<bf16>(v[3]).bits << 16);
            *reinterpret_cast<uint2*>((uint16_t*)p + i) = o;
        }
    } else {
        if (dt == ILM_DTYPE_F32) ((float*)p)[i] = v[0];
        else ((bf16*)p)[i] = from_f32<bf16>(v[0]);
    }
}

// NS: slots for streams (n of them are used)
template <int NS, int VEC, int THREADS>
__global__ void __launch_bounds__(THREADS)
hyper_update_kernel(void* __restrict__ x, float* __restrict__ X, const float* __restrict__ base, const void* __restrict__ y,
                    const float* __restrict__ mix, const float* __restrict__ outw, const float* __restrict__ inw,
                    const void* __restrict__ w, int n, int H, float alpha, float w_offset, float eps, int x_dt, int y_dt, int w_dt,
                    int parts, size_t part_stride, int write) {
    extern __shared__ __attribute__((aligned(16))) float urow[];     // H floats
    __shared__ float red[THREADS / 64];
    const int t = blockIdx.x, tid = threadIdx.x;
    const float* old = base != nullptr ? base + (size_t)t * H : X + (size_t)t * n * H;
    const size_t sstride = base != nullptr ? 0 : H;
    float* Xt = X + (size_t)t * n * H;
    float M[NS][NS], ow[NS], iw[NS];
#pragma unroll
    for (int s = 0; s < NS; ++s) {
        iw[s] = s < n ? (inw != nullptr ? inw[s] : 1.0f) : 0.f;
        ow[s] = (s < n && y != nullptr) ? outw[s] * alpha : 0.f;
#pragma unroll
        for (int q = 0; q < NS; ++q) M[s][q] = (s < n && q < n && y != nullptr) ? mix[s * n + q] : 0.f;
    }
    float ss = 0.f;
#pragma unroll 1
    for (int j = tid * VEC; j < H; j += THREADS * VEC) {
        float xs[NS][VEC], u[VEC];
#pragma unroll
        for (int s = 0; s < NS; ++s)
            if (s < n) hy_load<VEC>(old, s * sstride + j, ILM_DTYPE_F32, xs[s]);
#pragma unroll
        for (int e = 0; e < VEC; ++e) u[e] = 0.f;
        if (y != nullptr) {
            float yv[VEC];
#pragma unroll
            for (int e = 0; e < VEC; ++e) yv[e] = 0.f;
#pragma unroll 1
            for (int p0 = 0; p0 < parts; p0 += HY_PB) {
                float pv[HY_PB][VEC];
#pragma unroll
                for (int i = 0; i < HY_PB; ++i)
                    if (p0 + i < parts) hy_load<VEC>(y, (size_t)(p0 + i) * part_stride + (size_t)t * H + j, y_dt, pv[i]);
#pragma unroll
                for (int i = 0; i < HY_PB; ++i)
                    if (p0 + i < parts) {
#pragma unroll
                        for (int e = 0; e < VEC; ++e) yv[e] += pv[i][e];
                    }
            }
#pragma unroll
            for (int q = 0; q < NS; ++q)
                if (q < n) {
                    float xn[VEC];
#pragma unroll
                    for (int e = 0; e < VEC; ++e) xn[e] = ow[q] * yv[e];
#pragma unroll
                    for (int s = 0; s < NS; ++s)
                        if (s < n) {
#pragma unroll
                            for (int e = 0; e < VEC; ++e) xn[e] = fmaf(M[s][q], xs[s][e], xn[e]);
                        }
                    if (write) hy_store<VEC>(Xt, (size_t)q * H + j, ILM_DTYPE_F32, xn);
#pragma unroll
                    for (int e = 0; e < VEC; ++e) u[e] = fmaf(iw[q], xn[e], u[e]);
                }
        } else {
#pragma unroll
            for (int s = 0; s < NS; ++s)
                if (s < n) {
#pragma unroll
                    for (int e = 0; e < VEC; ++e) u[e] = fmaf(iw[s], xs[s][e], u[e]);
                }
        }
#pragma unroll
        for (int e = 0; e < VEC; ++e) {
            urow[j + e] = u[e];
            ss = fmaf(u[e], u[e], ss);
        }
    }
    if (x == nullptr) return;
    float rstd = 1.0f;
    if (w != nullptr) rstd = 1.0f / sqrtf(block_sum<THREADS / 64>(ss, red) / (float)H + eps);
#pragma unroll 1
    for (int j = tid * VEC; j < H; j += THREADS * VEC) {     // (a thread reads what it wrote itself)
        float o[VEC], wv[VEC];
        if (w != nullptr) hy_load<VEC>(w, j, w_dt, wv);
#pragma unroll
        for (int e = 0; e < VEC; ++e) o[e] = w != nullptr ? urow[j + e] * rstd * (wv[e] + w_offset) : urow[j + e];
        hy_store<VEC>(x, (size_t)t * H + j, x_dt, o);
    }
}

extern "C" int ilm_hyper_max_streams() { return HY_MAX_STREAMS; }
extern "C" int ilm_hyper_max_width() { return HY_MAX_H; }

extern "C" int ilm_hyper_update(void* x, void* X, const void* base, const void* y, const void* mix, const void* outw,
                                const void* inw, const void* w, int T_, int n, int H, float alpha, float w_offset, float eps,
                                int x_dt, int y_dt, int w_dt, int parts, long part_stride, int write, hipStream_t stream) {
    ILM_REQUIRE(T_ > 0 && n > 0 && H > 0, "hyper_update: bad sizes T=%d n=%d H=%d", T_, n, H);
    ILM_REQUIRE(n <= HY_MAX_STREAMS && H <= HY_MAX_H, "hyper_update: %d streams of %d, at most %d of %d", n, H, HY_MAX_STREAMS, HY_MAX_H);
    ILM_REQUIRE(y == nullptr || (mix != nullptr && outw != nullptr && parts >= 1), "hyper_update: a branch comes with its weights");
    ILM_REQUIRE(base != nullptr || X != nullptr, "hyper_update: no rows to read");
    ILM_REQUIRE(!write || (X != nullptr && y != nullptr), "hyper_update: nothing to write");
    ILM_REQUIRE(x_dt == ILM_DTYPE_F32 || x_dt == ILM_DTYPE_BF16, "hyper_update: unknown dtype %d", x_dt);
    const bool vec = H % 4 == 0 && part_stride % 4 == 0
                     && (((uintptr_t)x | (uintptr_t)X | (uintptr_t)base | (uintptr_t)y | (uintptr_t)w) & 15) == 0;
    const size_t shm = (size_t)H * sizeof(float);
    const bool wide = vec && H > 1024 && T_ <= 4 * ilm_num_cus();   // few rows: more waves a row
#define HY_ARGS x, (float*)X, (const float*)base, y, (const float*)mix, (const float*)outw, (const float*)inw, w, n, H, alpha, \
                w_offset, eps, x_dt, y_dt, w_dt, parts, (size_t)part_stride, write
#define HY_CASE(NS_)                                                                              \
    do {                                                                                          \
        if (wide) hyper_update_kernel<NS_, 4, 1024><<<T_, 1024, shm, stream>>>(HY_ARGS);          \
        else if (vec) hyper_update_kernel<NS_, 4, 256><<<T_, 256, shm, stream>>>(HY_ARGS);        \
        else hyper_update_kernel<NS_, 1, 256><<<T_, 256, shm, stream>>>(HY_ARGS);                 \
    } while (0)
    if (n <= 2) HY_CASE(2);
    else if (n <= 4) HY_CASE(4);
    else if (n <= 8) HY_CASE(8);
    else hyper_update_kernel<16, 1, 256><<<T_, 256, shm, stream>>>(HY_ARGS);
#undef HY_CASE
#undef HY_ARGS
    ILM_LAUNCH_CHECK("hyper_update");
    return 0;
}
