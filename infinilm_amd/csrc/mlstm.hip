// The matrix memory of an mLSTM: a linear attention whose state is written and forgotten through exponential gates, kept in
// range by a running maximum, and read through a denominator.  Per head, with the vectors of token t as rows and its log gates
//
//   li = cap tanh((raw_i + b_i) / cap),     lf = log sigmoid(cap tanh((raw_f + b_f) / cap))
//   m_t = max(lf + m_{t-1}, li)             (m_0 = 0)
//   S_t = exp(lf + m_{t-1} - m_t) S_{t-1} + exp(li - m_t) outer(k_t, v_t),      n_t likewise with k_t alone
//   o_t = q_t S_t / (max(|n_t . q_t|, exp(-m_t)) + 1e-6),                       q_t scaled by dk^(-1/2)
//
// and, where a block holds all columns of a head, y_t = o_t / sqrt(mean(o_t^2) + eps) * w * sigmoid(gate) in the activations'
// dtype.  Everything but the rows themselves is float.  Rows are those of one fused projection, [q: H dk | k: H dk | v: H dv | ...]
// with the raw gates and the output gate at offsets of their own.
//
// A request's state passes from step to step through rows of two pools, [H, dv + 1, dk] (the key index fastest; row dv is n) and
// [H] (m).
//
//   ilm_mlstm_step     token by token, a block a (request, head, columns).  A thread keeps ML_NK state entries of VC columns in
//       registers; the first wave keeps n as well, and n . q is folded with the columns' sums.
//
// (Long segments: mlstm_chunks.hip.)
#include "mlstm.h"

#define ML_NK 8

// (n and m are written back only where the block holds the whole head.)
// (128 registers: four waves a SIMD, two blocks of a head of 128 x 128 a compute unit)
template <typename T, int THREADS, int VC, bool NORM>
__global__ void __launch_bounds__(THREADS, 4)
mlstm_step_kernel(float* __restrict__ o, void* __restrict__ y, MlRows a, float* __restrict__ pool, float* __restrict__ pool_m,
                  const int* __restrict__ state_in, const int* __restrict__ state_out, const int* __restrict__ seg_offsets, int H, int dk,
                  int dv, int KP, int max_len, int y_stride, int y_dt) {
    __shared__ float red[THREADS / 64];
    __shared__ float den[2];
    const int h = blockIdx.y, r = blockIdx.z;
    const int t0 = seg_offsets[r], t1 = seg_offsets[r + 1];
    if (t0 >= t1 || t1 - t0 > max_len) return;       // (longer segments are another kernel's)
    int kp = threadIdx.x % KP, c0 = (blockIdx.x * (THREADS / KP) + threadIdx.x / KP) * VC;
    const bool with_n = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6) == 0;      // (every group of lanes of the first wave keeps n)
    const size_t hs = (size_t)dk * (dv + 1);
    const float* src = pool + ((size_t)state_in[r] * H + h) * hs;
    float m = pool_m[(size_t)state_in[r] * H + h];
    const bool v4 = dk % 4 == 0;
    // the thread's entries 4 p .. 4 p + 3 are k = kof[p] .. kof[p] + 3
    const int kof[2] = {4 * kp, 4 * (KP + kp)};
    // (a token's raw gates are loaded ahead: the first ones before the state, so that nothing waits for the state to form them)
    float zi, zf;
    ml_raw_gates<T>(a, t0, h, zi, zf);
    float S[VC][ML_NK], N[ML_NK];
    auto load_state = [&](float (&s)[ML_NK], int c) {      // column c of the state (dv: n)
#pragma unroll
        for (int p = 0; p < 2; ++p) {
            const bool ok = c <= dv && kof[p] < dk;
            const float* at = src + (size_t)(ok ? c : 0) * dk + (ok ? kof[p] : 0);
            if (v4) {
                const float4 t = ok ? *reinterpret_cast<const float4*>(at) : make_float4(0.f, 0.f, 0.f, 0.f);
                s[4 * p] = t.x; s[4 * p + 1] = t.y; s[4 * p + 2] = t.z; s[4 * p + 3] = t.w;
            } else {
#pragma unroll
                for (int e = 0; e < 4; ++e) s[4 * p + e] = (ok && kof[p] + e < dk) ? at[e] : 0.f;
            }
        }
    };
#pragma unroll
    for (int c = 0; c < VC; ++c) load_state(S[c], c0 + c < dv ? c0 + c : dv + 1);
    if (with_n) load_state(N, dv);
    const T* base = (const T*)a.rows;
    for (int t = t0; t < t1; ++t) {
        // (opaque: what follows from the lane's number would else be formed before the loop and held in registers)
        asm volatile("" : "+v"(kp), "+v"(c0));
        const int kof[2] = {4 * kp, 4 * (KP + kp)};
        const T* row = base + (size_t)t * a.stride;
        const T* qp = row + (size_t)h * dk;
        const T* kq = qp + (size_t)H * dk;
        const T* vp = row + (size_t)2 * H * dk + (size_t)h * dv;
        float q[ML_NK], k[ML_NK], v[VC];
#pragma unroll
        for (int p = 0; p < 2; ++p) {
            const bool in = kof[p] < dk;
            if (v4) {
                ml_ld4(qp + (in ? kof[p] : 0), q + 4 * p);
                ml_ld4(kq + (in ? kof[p] : 0), k + 4 * p);
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    q[4 * p + e] = in ? q[4 * p + e] : 0.f;
                    k[4 * p + e] = in ? k[4 * p + e] : 0.f;
                }
            } else {
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const bool ok = kof[p] + e < dk;
                    q[4 * p + e] = ok ? ml_ld(qp + kof[p] + e) : 0.f;
                    k[4 * p + e] = ok ? ml_ld(kq + kof[p] + e) : 0.f;
                }
            }
        }
#pragma unroll
        for (int c = 0; c < VC; ++c) v[c] = ml_ld(vp + (c0 + c < dv ? c0 + c : 0));
        float wg = 0.f, gg = 0.f;           // the norm's weight and the gate of the column this lane ends, on their way early
        if constexpr (NORM) {
            if (kp < VC && c0 + kp < dv) {
                wg = ml_any(a.norm_w, a.w_dt, h * dv + c0 + kp);
                gg = ml_ld(row + a.g_off + h * dv + c0 + kp);
            }
        }
        const float li = ml_capped(zi, a.cap), lf = ml_log_sigmoid(ml_capped(zf, a.cap));
        if (t + 1 < t1) ml_raw_gates<T>(a, t + 1, h, zi, zf);
        const float mn = fmaxf(lf + m, li), keep = expf(lf + m - mn), put = expf(li - mn);
        m = mn;
        float rq[VC];
#pragma unroll
        for (int c = 0; c < VC; ++c) {
            const float pv = put * v[c];
            rq[c] = 0.f;
#pragma unroll
            for (int i = 0; i < ML_NK; ++i) {
                S[c][i] = fmaf(k[i], pv, keep * S[c][i]);
                rq[c] = fmaf(S[c][i], q[i], rq[c]);
            }
        }
        float nq = 0.f;
        if (with_n) {
#pragma unroll
            for (int i = 0; i < ML_NK; ++i) {
                N[i] = fmaf(k[i], put, keep * N[i]);
                nq = fmaf(N[i], q[i], nq);
            }
            for (int off = 1; off < KP; off <<= 1) nq += __shfl_xor(nq, off, 64);
            if (threadIdx.x == 0) den[t & 1] = fmaxf(fabsf(nq * a.scale), expf(-m)) + 1e-6f;
        }
        for (int off = 1; off < KP; off <<= 1) {
#pragma unroll
            for (int c = 0; c < VC; ++c) rq[c] += __shfl_xor(rq[c], off, 64);
        }
        __syncthreads();
        const float to_o = a.scale / den[t & 1];
        float ov[VC];
#pragma unroll
        for (int c = 0; c < VC; ++c) ov[c] = rq[c] * to_o;
        if constexpr (NORM) {
            float ss = 0.f;
            if (kp == 0) {
#pragma unroll
                for (int c = 0; c < VC; ++c) ss = c0 + c < dv ? fmaf(ov[c], ov[c], ss) : ss;
            }
            const float rstd = 1.0f / sqrtf(block_sum<THREADS / 64>(ss, red) / (float)dv + a.eps);
#pragma unroll
            for (int c = 0; c < VC; ++c)
                if (kp == c % KP && c0 + c < dv) {      // (the columns' ends spread over the lanes)
                    const int j = h * dv + c0 + c;
                    if (c != kp) {      // (fewer lanes a column than columns a thread)
                        wg = ml_any(a.norm_w, a.w_dt, j);
                        gg = ml_ld(row + a.g_off + j);
                    }
                    const float z = ov[c] * rstd * wg * ml_sigmoid(gg);
                    if (y_dt == ILM_DTYPE_F32) ((float*)y)[(size_t)t * y_stride + j] = z;
                    else ((bf16*)y)[(size_t)t * y_stride + j] = from_f32<bf16>(z);
                }
        } else {
#pragma unroll
            for (int c = 0; c < VC; ++c)
                if (kp == c % KP && c0 + c < dv) o[((size_t)t * H + h) * dv + c0 + c] = ov[c];
        }
    }
    float* dst = pool + ((size_t)state_out[r] * H + h) * hs;
    auto store_state = [&](const float (&s)[ML_NK], int c) {
#pragma unroll
        for (int p = 0; p < 2; ++p) {
            float* at = dst + (size_t)c * dk + kof[p];
            if (v4) {
                if (kof[p] < dk) *reinterpret_cast<float4*>(at) = make_float4(s[4 * p], s[4 * p + 1], s[4 * p + 2], s[4 * p + 3]);
            } else {
#pragma unroll
                for (int e = 0; e < 4; ++e)
                    if (kof[p] + e < dk) at[e] = s[4 * p + e];
            }
        }
    };
#pragma unroll
    for (int c = 0; c < VC; ++c)
        if (c0 + c < dv) store_state(S[c], c0 + c);
    if (gridDim.x == 1 && threadIdx.x < KP) {
        store_state(N, dv);
        if (threadIdx.x == 0) pool_m[(size_t)state_out[r] * H + h] = m;
    }
}

// n and m of the heads whose columns are spread over several blocks of the step kernel (which all read the old ones): a block a
// (head, request), run after it.
template <typename T>
__global__ void __launch_bounds__(256)
mlstm_step_norms_kernel(MlRows a, float* __restrict__ pool, float* __restrict__ pool_m, const int* __restrict__ state_in,
                        const int* __restrict__ state_out, const int* __restrict__ seg_offsets, int H, int dk, int dv, int max_len) {
    const int h = blockIdx.x, r = blockIdx.y;
    const int t0 = seg_offsets[r], t1 = seg_offsets[r + 1];
    if (t0 >= t1 || t1 - t0 > max_len) return;
    const size_t hs = (size_t)dk * (dv + 1);
    const float* src = pool + ((size_t)state_in[r] * H + h) * hs + (size_t)dv * dk;
    float* dst = pool + ((size_t)state_out[r] * H + h) * hs + (size_t)dv * dk;
    const float m0 = pool_m[(size_t)state_in[r] * H + h];
    float m = m0;
    __syncthreads();
    for (int d0 = 0; d0 < dk; d0 += 256) {
        const int d = d0 + threadIdx.x;
        float n = d < dk ? src[d] : 0.f;
        m = m0;
        for (int t = t0; t < t1; ++t) {
            float li, lf;
            ml_gates<T>(a, t, h, li, lf);
            const float mn = fmaxf(lf + m, li), keep = expf(lf + m - mn), put = expf(li - mn);
            m = mn;
            if (d < dk) n = fmaf(ml_ld((const T*)a.rows + (size_t)t * a.stride + (size_t)(H + h) * dk + d), put, keep * n);
        }
        if (d < dk) dst[d] = n;
    }
    if (threadIdx.x == 0) pool_m[(size_t)state_out[r] * H + h] = m;
}

extern "C" int ilm_mlstm_max_dk() { return ML_NK * 64; }

static int ml_lanes(int dk) {
    int KP = 1;
    while (KP * ML_NK < dk) KP <<= 1;
    return KP;
}
// What a block of the step kernel must look like to hold a head's state whole: (threads, columns a thread), or 0.
static int ml_whole(int KP, int dv, int* threads, int* vc) {
    for (int th = 256; th <= 1024; th <<= 1)      // (four columns a thread leave four waves a SIMD their registers)
        for (int c = th == 256 ? 1 : 4; c <= 4; c <<= 1)
            if ((th / KP) * c >= dv) { *threads = th; *vc = c; return 1; }
    return 0;
}
// Whether the step kernel can end with the output norm (a block holds a head's state whole).
extern "C" int ilm_mlstm_step_norm_ok(int dk, int dv) {
    int th, vc;
    return dk <= ML_NK * 64 && ml_whole(ml_lanes(dk), dv, &th, &vc);
}

// y != null: with the output norm (see ilm_mlstm_step_norm_ok); else o [T, H dv] float.  Segments of more than max_len tokens are
// passed over.
extern "C" int ilm_mlstm_step(void* o, void* y, const void* rows, int row_stride, int rows_dt, const void* bias_i, const void* bias_f, int b_dt,
                              int i_off, int f_off, int g_off, float cap, float scale, void* pool, void* pool_m, const void* state_in,
                              const void* state_out, const void* seg_offsets, int R, int H, int dk, int dv, int max_len, const void* norm_w, int w_dt,
                              float eps, int y_stride, int y_dt, hipStream_t stream) {
    ML_CHECK_ROWS("mlstm_step");
    ILM_REQUIRE(dk <= ML_NK * 64, "mlstm_step: keys of %d, at most %d", dk, ML_NK * 64);
    ILM_REQUIRE((y != nullptr) != (o != nullptr), "mlstm_step: one kind of result");
    const int KP = ml_lanes(dk);
#define ML_ARGS (float*)o, y, a, (float*)pool, (float*)pool_m, (const int*)state_in, (const int*)state_out, (const int*)seg_offsets, H, dk, dv,  \
                KP, max_len, y_stride, y_dt
#define ML_T(TH_, VC_, N_, GRID_)                                                                                                      \
    {                                                                                                                                  \
        if (rows_dt == ILM_DTYPE_F32) mlstm_step_kernel<float, TH_, VC_, N_><<<GRID_, TH_, 0, stream>>>(ML_ARGS);                       \
        else mlstm_step_kernel<bf16, TH_, VC_, N_><<<GRID_, TH_, 0, stream>>>(ML_ARGS);                                                 \
    }
    if (y != nullptr) {
        int th = 0, vc = 0;
        ILM_REQUIRE(ml_whole(KP, dv, &th, &vc), "mlstm_step: a head's state of %d x %d does not fit a block", dk, dv);
        const dim3 grid(1, H, R);
        if (th == 256 && vc == 1) ML_T(256, 1, true, grid)
        else if (th == 256 && vc == 2) ML_T(256, 2, true, grid)
        else if (th == 256) ML_T(256, 4, true, grid)
        else if (th == 512) ML_T(512, 4, true, grid)
        else ML_T(1024, 4, true, grid)
        ILM_LAUNCH_CHECK("mlstm_step (with the output norm)");
        return 0;
    }
    const int per = 256 / KP * 4;
    const int blocks = (dv + per - 1) / per;
    const dim3 grid(blocks, H, R);
    ML_T(256, 4, false, grid)
    ILM_LAUNCH_CHECK("mlstm_step");
    if (blocks > 1) {
        if (rows_dt == ILM_DTYPE_F32)
            mlstm_step_norms_kernel<float><<<dim3(H, R), 256, 0, stream>>>(a, (float*)pool, (float*)pool_m, (const int*)state_in, (const int*)state_out,
                                                                           (const int*)seg_offsets, H, dk, dv, max_len);
        else
            mlstm_step_norms_kernel<bf16><<<dim3(H, R), 256, 0, stream>>>(a, (float*)pool, (float*)pool_m, (const int*)state_in, (const int*)state_out,
                                                                          (const int*)seg_offsets, H, dk, dv, max_len);
        ILM_LAUNCH_CHECK("mlstm_step (norms)");
    }
#undef ML_T
#undef ML_ARGS
    return 0;
}
