// The gated delta rule: a linear attention whose state forgets by a decay per head and step and is corrected by the
// difference between a token's value and what the state already holds under the token's key.  Per head, all in float:
//
//   S <- g S;   u = beta (v - S^T k);   S <- S + k u^T;   o = S^T q            S [dk, dv], zero at a sequence's start
//
// Inputs are float rows [q: G dkp | k: G dkp | v: H dv] (query and key heads filled up with zeros to dkp entries; head h reads
// query/key head h / (H / G)) and [beta: H | log g: H].  A request's state passes from step to step through a row of a pool,
// [H, dv, dk] (the key index fastest).
//
//   ilm_delta_step     token by token, a block a (request, head, columns).  A thread keeps DS_NK consecutive state entries
//       of VC value columns in registers; the two sums a token needs, S^T k and S^T q (both from the decayed state: the
//       read-out after the write is S^T q + u (k . q)), and k . q are folded over the lanes of a column together.  Where a block
//       holds all columns of its head it can end with the head's output norm, weight and gate:
//       y = o / sqrt(mean(o^2) + eps) * w * silu(gate), in the activations' dtype.
#include "common.h"

#define DS_NK 8

template <int THREADS, int VC, bool NORM>
__global__ void __launch_bounds__(THREADS)
delta_step_kernel(float* __restrict__ o, void* __restrict__ y, const float* __restrict__ rows, int row_stride,
                  const float* __restrict__ gates, float* __restrict__ pool, const int* __restrict__ state_in,
                  const int* __restrict__ state_out, const int* __restrict__ seg_offsets, int H, int G, int dk, int dkp, int dv, int KP,
                  int max_len, const void* __restrict__ norm_w, const void* __restrict__ gate, int gate_stride, float eps, int y_stride,
                  int y_dt, int w_dt, int gate_dt) {
    __shared__ float red[THREADS / 64];
    const int h = blockIdx.y, r = blockIdx.z;
    const int t0 = seg_offsets[r], t1 = seg_offsets[r + 1];
    if (t0 >= t1 || t1 - t0 > max_len) return;       // (longer segments are another kernel's)
    const int kp = threadIdx.x % KP, c0 = (blockIdx.x * (THREADS / KP) + threadIdx.x / KP) * VC, k0 = kp * DS_NK;
    const size_t hs = (size_t)dk * dv;
    const float* src = pool + ((size_t)state_in[r] * H + h) * hs;
    const bool v4 = dk % 4 == 0;
    float S[VC][DS_NK];
#pragma unroll
    for (int c = 0; c < VC; ++c) {
#pragma unroll
        for (int i = 0; i < DS_NK; i += 4) {
            const bool ok = c0 + c < dv && k0 + i < dk;
            const float* p = src + (size_t)(c0 + c) * dk + k0 + i;
            if (v4) {
                const float4 t = ok ? *reinterpret_cast<const float4*>(p) : make_float4(0.f, 0.f, 0.f, 0.f);
                S[c][i] = t.x; S[c][i + 1] = t.y; S[c][i + 2] = t.z; S[c][i + 3] = t.w;
            } else {
#pragma unroll
                for (int e = 0; e < 4; ++e) S[c][i + e] = (ok && k0 + i + e < dk) ? p[e] : 0.f;
            }
        }
    }
    const int g = h / (H / G);
    const bool kin = k0 < dkp;                          // (dkp is a multiple of 8: a thread's entries all lie inside, or none does)
    const float* qp = rows + (size_t)g * dkp + (kin ? k0 : 0);
    const float* kq = qp + (size_t)G * dkp;
    const float* vp = rows + (size_t)2 * G * dkp + (size_t)h * dv;
    for (int t = t0; t < t1; ++t) {
        float q[DS_NK], k[DS_NK], v[VC];
#pragma unroll
        for (int i = 0; i < DS_NK; i += 4) {
            const float4 a = *reinterpret_cast<const float4*>(qp + (size_t)t * row_stride + i);
            const float4 b = *reinterpret_cast<const float4*>(kq + (size_t)t * row_stride + i);
            q[i] = kin ? a.x : 0.f; q[i + 1] = kin ? a.y : 0.f; q[i + 2] = kin ? a.z : 0.f; q[i + 3] = kin ? a.w : 0.f;
            k[i] = kin ? b.x : 0.f; k[i + 1] = kin ? b.y : 0.f; k[i + 2] = kin ? b.z : 0.f; k[i + 3] = kin ? b.w : 0.f;
        }
#pragma unroll
        for (int c = 0; c < VC; ++c) v[c] = vp[(size_t)t * row_stride + (c0 + c < dv ? c0 + c : 0)];
        const float beta = gates[(size_t)t * 2 * H + h], dec = expf(gates[(size_t)t * 2 * H + H + h]);
        float rk[VC], rq[VC], kdq = 0.f;
#pragma unroll
        for (int i = 0; i < DS_NK; ++i) kdq = fmaf(k[i], q[i], kdq);
#pragma unroll
        for (int c = 0; c < VC; ++c) {
            rk[c] = 0.f;
            rq[c] = 0.f;
#pragma unroll
            for (int i = 0; i < DS_NK; ++i) {
                S[c][i] *= dec;
                rk[c] = fmaf(S[c][i], k[i], rk[c]);
                rq[c] = fmaf(S[c][i], q[i], rq[c]);
            }
        }
        for (int off = 1; off < KP; off <<= 1) {
            kdq += __shfl_xor(kdq, off, 64);
#pragma unroll
            for (int c = 0; c < VC; ++c) {
                rk[c] += __shfl_xor(rk[c], off, 64);
                rq[c] += __shfl_xor(rq[c], off, 64);
            }
        }
        float ov[VC];
#pragma unroll
        for (int c = 0; c < VC; ++c) {
            const float u = beta * (v[c] - rk[c]);
            ov[c] = fmaf(u, kdq, rq[c]);
#pragma unroll
            for (int i = 0; i < DS_NK; ++i) S[c][i] = fmaf(k[i], u, S[c][i]);
        }
        if constexpr (NORM) {
            float ss = 0.f;
            if (kp == 0) {
#pragma unroll
                for (int c = 0; c < VC; ++c) ss = c0 + c < dv ? fmaf(ov[c], ov[c], ss) : ss;
            }
            const float rstd = 1.0f / sqrtf(block_sum<THREADS / 64>(ss, red) / (float)dv + eps);
#pragma unroll
            for (int c = 0; c < VC; ++c)
                if (kp == c % KP && c0 + c < dv) {      // (the columns' ends spread over the lanes)
                    const int j = c0 + c;
                    const float gv = gate_dt == ILM_DTYPE_F32 ? ((const float*)gate)[(size_t)t * gate_stride + h * dv + j]
                                                              : to_f32(((const bf16*)gate)[(size_t)t * gate_stride + h * dv + j]);
                    const float wv = w_dt == ILM_DTYPE_F32 ? ((const float*)norm_w)[j] : to_f32(((const bf16*)norm_w)[j]);
                    const float z = ov[c] * rstd * wv * (gv / (1.0f + expf(-gv)));
                    if (y_dt == ILM_DTYPE_F32) ((float*)y)[(size_t)t * y_stride + h * dv + j] = z;
                    else ((bf16*)y)[(size_t)t * y_stride + h * dv + j] = from_f32<bf16>(z);
                }
        } else {
#pragma unroll
            for (int c = 0; c < VC; ++c)
                if (kp == c % KP && c0 + c < dv) o[((size_t)t * H + h) * dv + c0 + c] = ov[c];
        }
    }
    float* dst = pool + ((size_t)state_out[r] * H + h) * hs;
#pragma unroll
    for (int c = 0; c < VC; ++c)
        if (c0 + c < dv) {
#pragma unroll
            for (int i = 0; i < DS_NK; i += 4) {
                float* p = dst + (size_t)(c0 + c) * dk + k0 + i;
                if (v4) {
                    if (k0 + i < dk) *reinterpret_cast<float4*>(p) = make_float4(S[c][i], S[c][i + 1], S[c][i + 2], S[c][i + 3]);
                } else {
#pragma unroll
                    for (int e = 0; e < 4; ++e)
                        if (k0 + i + e < dk) p[e] = S[c][i + e];
                }
            }
        }
}

extern "C" int ilm_delta_max_dk() { return DS_NK * 64; }

// What a block of the step kernel must look like to hold a head's [dk, dv] state whole: (threads, columns a thread), or 0.
static int ds_whole(int KP, int dv, int* threads, int* vc) {
    for (int th = 256; th <= 1024; th <<= 1)      // (four columns a thread leave four waves a SIMD their registers)
        for (int c = th == 256 ? 1 : 4; c <= 4; c <<= 1)
            if ((th / KP) * c >= dv) { *threads = th; *vc = c; return 1; }
    return 0;
}
static int ds_lanes(int dk) {
    int KP = 1;
    while (KP * DS_NK < dk) KP <<= 1;
    return KP;
}

// Whether the step kernel can end with the output norm (a block holds a head's state whole).
extern "C" int ilm_delta_step_norm_ok(int dk, int dv) {
    int th, vc;
    return dk <= DS_NK * 64 && ds_whole(ds_lanes(dk), dv, &th, &vc);
}

// y != null: with the output norm (see ilm_delta_step_norm_ok); else o [T, H dv] float.  Segments of more than max_len tokens are
// passed over.
extern "C" int ilm_delta_step(void* o, void* y, const void* rows, int row_stride, const void* gates, void* pool, const void* state_in,
                              const void* state_out, const void* seg_offsets, int R, int H, int G, int dk, int dkp, int dv, int max_len,
                              const void* norm_w, const void* gate, int gate_stride, float eps, int y_stride, int y_dt, int w_dt, int gate_dt,
                              hipStream_t stream) {
    ILM_REQUIRE(R > 0 && R <= 65535 && H > 0 && H <= 65535 && G > 0 && H % G == 0 && dk > 0 && dv > 0, "delta_step: bad sizes");
    ILM_REQUIRE(dk <= DS_NK * 64 && dkp >= dk && dkp % 8 == 0, "delta_step: keys of %d in %d, at most %d", dk, dkp, DS_NK * 64);
    ILM_REQUIRE(row_stride % 4 == 0 && ((uintptr_t)rows & 15) == 0 && ((uintptr_t)pool & 15) == 0, "delta_step: rows must be 16-byte aligned");
    ILM_REQUIRE((y != nullptr) != (o != nullptr), "delta_step: one kind of result");
    const int KP = ds_lanes(dk);
#define DS_ARGS (float*)o, y, (const float*)rows, row_stride, (const float*)gates, (float*)pool, (const int*)state_in,               \
                (const int*)state_out, (const int*)seg_offsets, H, G, dk, dkp, dv, KP, max_len, norm_w, gate, gate_stride, eps,      \
                y_stride, y_dt, w_dt, gate_dt
    if (y != nullptr) {
        int th = 0, vc = 0;
        ILM_REQUIRE(ds_whole(KP, dv, &th, &vc), "delta_step: a head's state of %d x %d does not fit a block", dk, dv);
        ILM_REQUIRE(norm_w != nullptr && gate != nullptr, "delta_step: the output norm needs its weight and the gate rows");
        const dim3 grid(1, H, R);
#define DS_N(TH_, VC_) if (th == TH_ && vc == VC_) delta_step_kernel<TH_, VC_, true><<<grid, TH_, 0, stream>>>(DS_ARGS)
        DS_N(256, 1); DS_N(256, 2); DS_N(256, 4); DS_N(512, 4); DS_N(1024, 4);
#undef DS_N
        ILM_LAUNCH_CHECK("delta_step (with the output norm)");
        return 0;
    }
    const int VT = 256 / KP;
    const int g4 = (dv + 4 * VT - 1) / (4 * VT);
    if ((long)g4 * H * R >= 2L * ilm_num_cus()) delta_step_kernel<256, 4, false><<<dim3(g4, H, R), 256, 0, stream>>>(DS_ARGS);
    else delta_step_kernel<256, 1, false><<<dim3((dv + VT - 1) / VT, H, R), 256, 0, stream>>>(DS_ARGS);
#undef DS_ARGS
    ILM_LAUNCH_CHECK("delta_step");
    return 0;
}
