// From the rows of a fused projection to what a mixer with short causal convolutions works on, in one kernel a step: the
// convolution over the tokens of each request per channel,
//   y[t, c] = sum_i w[i, c] x[t - (taps - 1) + i, c]     (the last tap is the token's own input; what lies before a request's
//                                                         first token of this step comes from its state row, zeros at first)
// and what follows it token by token:
//
//   ilm_conv_delta_inputs   rows [q: G dk | k: G dk | v: H dv | ...], y through silu; every q and k head divided by its length,
//       x / sqrt(sum(x^2) + unit_eps), q times q_scale; and from the rows' columns b and a [H each] the step's
//       beta = sigmoid(b) and log-decay = -exp(A_log) softplus(a + dt_bias).  Float results: rows [q | k | v] whose q and k heads
//       are filled up with zeros to dkp entries, and [T, 2 H] (beta | log-decay).
//   ilm_conv_norm_rope_kvwrite   rows [q: H dim | k: G dim | v: G vdim] (or q alone), q and k each RMS-normed over the whole
//       row of all their heads with a weight, the first rd entries of every head turned in the pairs (2i, 2i + 1) by position
//       x freq[i]; q goes out as heads of d entries (zeros beyond dim), k and v into the paged cache.
//
// A block a token; all arithmetic is float.  A request's state row holds its last taps - 1 inputs, oldest first.  The block of a
// request's only token of the step shifts the row itself (a thread touches its own channels); where requests bring more
// tokens, a second launch writes their rows from the old row and the step's inputs.
#include "common.h"

#define CP_MAX_TAPS 8
#define CP_MAX_LDS (64 * 1024)

template <int VEC, typename T>
__device__ __forceinline__ void cp_load(const T* p, float (&v)[VEC]) {
    if constexpr (VEC == 8 && sizeof(T) == 2) {
        const uint4 t = *reinterpret_cast<const uint4*>(p);
        v[0] = __uint_as_float(t.x << 16); v[1] = __uint_as_float(t.x & 0xffff0000u);
        v[2] = __uint_as_float(t.y << 16); v[3] = __uint_as_float(t.y & 0xffff0000u);
        v[4] = __uint_as_float(t.z << 16); v[5] = __uint_as_float(t.z & 0xffff0000u);
        v[6] = __uint_as_float(t.w << 16); v[7] = __uint_as_float(t.w & 0xffff0000u);
    } else if constexpr (VEC == 8) {
        const float4 a = *reinterpret_cast<const float4*>(p), b = *reinterpret_cast<const float4*>(p + 4);
        v[0] = a.x; v[1] = a.y; v[2] = a.z; v[3] = a.w; v[4] = b.x; v[5] = b.y; v[6] = b.z; v[7] = b.w;
    } else {
        v[0] = to_f32(*p);
    }
}
template <int VEC, typename T>
__device__ __forceinline__ void cp_store(T* p, const float (&v)[VEC]) {
    if constexpr (VEC == 8 && sizeof(T) == 2) {
        T o[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) o[e] = from_f32<T>(v[e]);
        *reinterpret_cast<uint4*>(p) = *reinterpret_cast<uint4*>(o);
    } else if constexpr (VEC == 8) {
        *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
        *reinterpret_cast<float4*>(p + 4) = make_float4(v[4], v[5], v[6], v[7]);
    } else {
        *p = from_f32<T>(v[0]);
    }
}

// x * sigmoid(x) on the hardware's exponential and reciprocal (each within an ulp)
__device__ __forceinline__ float cp_silu(float x) { return x * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-1.4426950408889634f * x)); }

// Blocks go to the eight dies in turn: with this numbering a die takes a run of consecutive tokens, whose convolutions read
// the same rows.  A grid of cp_blocks(T) blocks; block numbers beyond the last token give -1.
__device__ __forceinline__ int cp_token(int T_) {
    const int per = (T_ + 7) / 8, t = (int)(blockIdx.x & 7) * per + (int)(blockIdx.x >> 3);
    return (int)(blockIdx.x >> 3) < per && t < T_ ? t : -1;
}

static inline unsigned cp_blocks(int T_) { return 8u * (unsigned)((T_ + 7) / 8); }

// What a block needs to know of its token's request
struct cp_place {
    int j;              // the token's place in its segment
    bool only;          // the segment has no other token in this step
    const float* in;    // state row read (taps - 1 rows of C)
    float* out;         // state row written
};
__device__ __forceinline__ cp_place cp_find(int t, const int* seg, const int* seg_offsets, const int* state_in, const int* state_out,
                                            float* pool, int taps, int C) {
    const int r = seg[t];
    cp_place p;
    p.j = t - seg_offsets[r];
    p.only = seg_offsets[r + 1] - seg_offsets[r] == 1;
    p.in = taps > 1 ? pool + (size_t)state_in[r] * (taps - 1) * C : nullptr;
    p.out = taps > 1 ? pool + (size_t)state_out[r] * (taps - 1) * C : nullptr;
    return p;
}

// y of channels c .. c + VEC - 1, and the shift of the state row where the token is its segment's only one
template <int VEC, typename T, int MT>     // MT: the most taps
__device__ __forceinline__ void cp_conv(float (&y)[VEC], const T* x, int x_stride, const T* w, int t, int c, int C, int taps,
                                        const cp_place& p) {
    float own[VEC];
    cp_load<VEC, T>(x + (size_t)t * x_stride + c, own);
    if (taps == 0) {
#pragma unroll
        for (int e = 0; e < VEC; ++e) y[e] = own[e];
        return;
    }
    float xv[MT][VEC];
#pragma unroll
    for (int i = 0; i < MT - 1; ++i)
        if (i < taps - 1) {
            const int back = taps - 1 - i;
            if (back <= p.j) cp_load<VEC, T>(x + (size_t)(t - back) * x_stride + c, xv[i]);
            else cp_load<VEC, float>(p.in + (size_t)(taps - 1 - (back - p.j)) * C + c, xv[i]);
        }
#pragma unroll
    for (int e = 0; e < VEC; ++e) y[e] = 0.f;
#pragma unroll
    for (int i = 0; i < MT; ++i)
        if (i < taps) {
            float wv[VEC];
            cp_load<VEC, T>(w + (size_t)i * C + c, wv);
#pragma unroll
            for (int e = 0; e < VEC; ++e) y[e] = fmaf(wv[e], i == taps - 1 ? own[e] : xv[i < MT - 1 ? i : 0][e], y[e]);
        }
    if (p.only && taps > 1) {
#pragma unroll
        for (int i = 0; i < MT - 1; ++i)
            if (i < taps - 1) cp_store<VEC, float>(p.out + (size_t)i * C + c, i == taps - 2 ? own : xv[i + 1 < MT ? i + 1 : 0]);
    }
}

// the state rows of the segments of two and more tokens: entry i is the input taps - 1 - i tokens before the segment's end
template <typename T>
__global__ void __launch_bounds__(256)
conv_state_kernel(const T* __restrict__ x, float* __restrict__ pool, const int* __restrict__ state_in, const int* __restrict__ state_out,
                  const int* __restrict__ seg_offsets, int C, int taps, int x_stride) {
    const int r = blockIdx.y, c = blockIdx.x * 256 + threadIdx.x;
    if (c >= C) return;
    const int t0 = seg_offsets[r], len = seg_offsets[r + 1] - t0;
    if (len <= 1) return;
    const size_t sin = (size_t)state_in[r] * (taps - 1) * C, sout = (size_t)state_out[r] * (taps - 1) * C;
    float win[CP_MAX_TAPS];
#pragma unroll
    for (int i = 0; i < CP_MAX_TAPS; ++i) {
        const int back = taps - 1 - i;
        win[i] = 0.f;
        if (i < taps - 1) win[i] = back <= len ? to_f32(x[(size_t)(t0 + len - back) * x_stride + c]) : pool[sin + (size_t)(i + len) * C + c];
    }
#pragma unroll
    for (int i = 0; i < CP_MAX_TAPS; ++i)
        if (i < taps - 1) pool[sout + (size_t)i * C + c] = win[i];
}

template <typename T>
static int cp_state(const void* x, void* pool, const void* state_in, const void* state_out, const void* seg_offsets, int R, int C,
                    int taps, int x_stride, hipStream_t stream) {
    conv_state_kernel<T><<<dim3((C + 255) / 256, R), 256, 0, stream>>>((const T*)x, (float*)pool, (const int*)state_in,
                                                                       (const int*)state_out, (const int*)seg_offsets, C, taps, x_stride);
    ILM_LAUNCH_CHECK("conv_state");
    return 0;
}

// ------------------------------------------------------------------------------------------
template <int VEC, typename T, int THREADS>
__global__ void __launch_bounds__(THREADS)
conv_delta_inputs_kernel(float* __restrict__ out, float* __restrict__ gates, const T* __restrict__ x, const T* __restrict__ w,
                         float* __restrict__ pool, const int* __restrict__ state_in, const int* __restrict__ state_out,
                         const int* __restrict__ seg, const int* __restrict__ seg_offsets, const float* __restrict__ a_log,
                         const float* __restrict__ dt_bias, int T_, int H, int G, int dk, int dkp, int dv, int taps, int x_stride,
                         int out_stride, int b_off, int a_off, float q_scale, float unit_eps) {
    extern __shared__ __attribute__((aligned(16))) float qk[];     // 2 G dk
    const int t = cp_token(T_);
    if (t < 0) return;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int nqk = 2 * G * dk, C = nqk + H * dv;
    const cp_place p = cp_find(t, seg, seg_offsets, state_in, state_out, pool, taps, C);
    float* orow = out + (size_t)t * out_stride;
    for (int c = tid * VEC; c < C; c += THREADS * VEC) {
        float y[VEC];
        cp_conv<VEC, T, CP_MAX_TAPS>(y, x, x_stride, w, t, c, C, taps, p);
#pragma unroll
        for (int e = 0; e < VEC; ++e) y[e] = cp_silu(y[e]);
        if (c < nqk) {
            cp_store<VEC, float>(qk + c, y);
        } else {
            cp_store<VEC, float>(orow + 2 * G * dkp + (c - nqk), y);
        }
    }
    for (int h = tid; h < H; h += THREADS) {
        const float b = to_f32(x[(size_t)t * x_stride + b_off + h]);
        const float z = to_f32(x[(size_t)t * x_stride + a_off + h]) + dt_bias[h];
        const float sp = z > 20.0f ? z : log1pf(expf(z));
        gates[(size_t)t * 2 * H + h] = 1.0f / (1.0f + expf(-b));
        gates[(size_t)t * 2 * H + H + h] = -expf(a_log[h]) * sp;
    }
    __syncthreads();
    for (int u = wave; u < 2 * G; u += THREADS / 64) {
        float ss = 0.f;
        for (int e = lane; e < dk; e += 64) ss = fmaf(qk[u * dk + e], qk[u * dk + e], ss);
        const float f = (u < G ? q_scale : 1.0f) / sqrtf(wave_sum(ss) + unit_eps);
        for (int e = lane; e < dkp; e += 64) orow[u * dkp + e] = e < dk ? qk[u * dk + e] * f : 0.f;
    }
}

// The same without LDS where a head is a power of two of pieces of 8 entries (keys of 16 to 512), convolutions of 1 to 4 taps: a
// thread keeps the taps of its 8 channels and walks TB consecutive tokens, whose rows are all on their way from the start; a
// head's sum of squares is folded over its lanes.
template <typename T, int TB, int TAPS>
__global__ void __launch_bounds__(256)
conv_delta_inputs_fast_kernel(float* __restrict__ out, float* __restrict__ gates, const T* __restrict__ x, const T* __restrict__ w,
                              float* __restrict__ pool, const int* __restrict__ state_in, const int* __restrict__ state_out,
                              const int* __restrict__ seg, const int* __restrict__ seg_offsets, const float* __restrict__ a_log,
                              const float* __restrict__ dt_bias, int T_, int H, int G, int dk, int dv, int x_stride, int out_stride,
                              int b_off, int a_off, float q_scale, float unit_eps) {
    const int grp = cp_token((T_ + TB - 1) / TB);
    if (grp < 0) return;
    const int tb = grp * TB;
    const int nqk = 2 * G * dk, C = nqk + H * dv, lanes = dk >> 3;
    if (blockIdx.y == 0)
        for (int i = threadIdx.x; i < TB * H; i += 256) {
            const int t = tb + i / H, h = i % H;
            if (t >= T_) break;
            const float b = to_f32(x[(size_t)t * x_stride + b_off + h]);
            const float z = to_f32(x[(size_t)t * x_stride + a_off + h]) + dt_bias[h];
            const float sp = z > 20.0f ? z : log1pf(expf(z));
            gates[(size_t)t * 2 * H + h] = 1.0f / (1.0f + expf(-b));
            gates[(size_t)t * 2 * H + H + h] = -expf(a_log[h]) * sp;
        }
    const int c = (blockIdx.y * 256 + threadIdx.x) * 8;
    if (c >= C) return;                     // (values' lanes: no head's sum misses them)
    float own[TB][8], wv[TAPS][8];
#pragma unroll
    for (int i = 0; i < TB; ++i) cp_load<8, T>(x + (size_t)(tb + i < T_ ? tb + i : T_ - 1) * x_stride + c, own[i]);
#pragma unroll
    for (int i = 0; i < TAPS; ++i) cp_load<8, T>(w + (size_t)i * C + c, wv[i]);
    float win[TAPS > 1 ? TAPS - 1 : 1][8];
#pragma unroll
    for (int i = 0; i < TB; ++i) {
        const int t = tb + i;
        if (t >= T_) return;
        const cp_place p = cp_find(t, seg, seg_offsets, state_in, state_out, pool, TAPS, C);
        if constexpr (TAPS > 1) {
            if (i == 0 || p.j == 0) {
#pragma unroll
                for (int m = 0; m < TAPS - 1; ++m) {
                    const int back = TAPS - 1 - m;
                    if (back <= p.j) cp_load<8, T>(x + (size_t)(t - back) * x_stride + c, win[m]);
                    else cp_load<8, float>(p.in + (size_t)(TAPS - 1 - (back - p.j)) * C + c, win[m]);
                }
            }
        }
        float y[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            y[e] = 0.f;
#pragma unroll
            for (int m = 0; m < TAPS - 1; ++m) y[e] = fmaf(wv[m][e], win[m][e], y[e]);
            y[e] = cp_silu(fmaf(wv[TAPS - 1][e], own[i][e], y[e]));
        }
        if (c < nqk) {                      // (the lanes of a head agree)
            float ss = 0.f;
#pragma unroll
            for (int e = 0; e < 8; ++e) ss = fmaf(y[e], y[e], ss);
            for (int off = 1; off < lanes; off <<= 1) ss += __shfl_xor(ss, off, 64);
            const float f = (c < G * dk ? q_scale : 1.0f) / sqrtf(ss + unit_eps);
#pragma unroll
            for (int e = 0; e < 8; ++e) y[e] *= f;
        }
        cp_store<8, float>(out + (size_t)t * out_stride + c, y);
        if constexpr (TAPS > 1) {
#pragma unroll
            for (int m = 0; m < TAPS - 1; ++m) {
#pragma unroll
                for (int e = 0; e < 8; ++e) win[m][e] = m + 1 < TAPS - 1 ? win[m + 1 < TAPS - 1 ? m + 1 : 0][e] : own[i][e];
                if (p.only) cp_store<8, float>(p.out + (size_t)m * C + c, win[m]);
            }
        }
    }
}

extern "C" int ilm_conv_prep_max_taps() { return CP_MAX_TAPS; }

// `singles`: every segment brings one token at most (the state rows are then all shifted by the blocks themselves).
extern "C" int ilm_conv_delta_inputs(void* out, void* gates, const void* x, const void* w, void* pool, const void* state_in,
                                     const void* state_out, const void* seg, const void* seg_offsets, const void* a_log,
                                     const void* dt_bias, int T_, int R, int H, int G, int dk, int dkp, int dv, int taps, int x_stride,
                                     int out_stride, int b_off, int a_off, float q_scale, float unit_eps, int singles, int dtype,
                                     hipStream_t stream) {
    const int nqk = 2 * G * dk, C = nqk + H * dv;
    ILM_REQUIRE(T_ > 0 && R > 0 && R <= 65535 && H > 0 && G > 0 && H % G == 0 && dk > 0 && dkp >= dk && dv > 0, "conv_delta_inputs: bad sizes");
    ILM_REQUIRE(taps >= 0 && taps <= CP_MAX_TAPS, "conv_delta_inputs: %d taps, at most %d", taps, CP_MAX_TAPS);
    ILM_REQUIRE(taps <= 1 || pool != nullptr, "conv_delta_inputs: a convolution needs its state rows");
    ILM_REQUIRE(taps == 0 || w != nullptr, "conv_delta_inputs: a convolution needs its weights");
    ILM_REQUIRE((size_t)nqk * 4 <= CP_MAX_LDS, "conv_delta_inputs: %d query and key channels, at most %d", nqk, CP_MAX_LDS / 4);
    ILM_REQUIRE(out_stride >= 2 * G * dkp + H * dv && b_off + H <= x_stride && a_off + H <= x_stride, "conv_delta_inputs: rows too short");
    const bool vec = dk % 4 == 0 && (G * dk) % 4 == 0 && nqk % 8 == 0 && C % 8 == 0 && x_stride % 8 == 0 && out_stride % 4 == 0 && (2 * G * dkp) % 4 == 0
                     && (((uintptr_t)x | (uintptr_t)w | (uintptr_t)pool | (uintptr_t)out) & 15) == 0;
    const bool wide = T_ <= 2 * ilm_num_cus();
    const bool fast = vec && dk == dkp && (dk & (dk - 1)) == 0 && dk >= 16 && dk <= 512 && dv % 8 == 0 && taps >= 1 && taps <= 4;
    if (fast) {
        const int TB = T_ >= 8 * 64 ? 8 : 1;
        const dim3 grid(cp_blocks((T_ + TB - 1) / TB), (C / 8 + 255) / 256);
#define CF_ARGS(T__) (float*)out, (float*)gates, (const T__*)x, (const T__*)w, (float*)pool, (const int*)state_in, (const int*)state_out, \
                     (const int*)seg, (const int*)seg_offsets, (const float*)a_log, (const float*)dt_bias, T_, H, G, dk, dv, x_stride,  \
                     out_stride, b_off, a_off, q_scale, unit_eps
#define CF_TAPS(T__, TAPS_)                                                                                                          \
    case TAPS_:                                                                                                                      \
        if (TB == 8) conv_delta_inputs_fast_kernel<T__, 8, TAPS_><<<grid, 256, 0, stream>>>(CF_ARGS(T__));                           \
        else conv_delta_inputs_fast_kernel<T__, 1, TAPS_><<<grid, 256, 0, stream>>>(CF_ARGS(T__));                                   \
        break
        if (dtype == ILM_DTYPE_F32) {
            switch (taps) { CF_TAPS(float, 1); CF_TAPS(float, 2); CF_TAPS(float, 3); CF_TAPS(float, 4); }
        } else if (dtype == ILM_DTYPE_BF16) {
            switch (taps) { CF_TAPS(bf16, 1); CF_TAPS(bf16, 2); CF_TAPS(bf16, 3); CF_TAPS(bf16, 4); }
        } else {
            ILM_REQUIRE(false, "conv_delta_inputs: unknown dtype %d", dtype);
        }
#undef CF_TAPS
#undef CF_ARGS
    } else {
#define CD_ARGS(T__) (float*)out, (float*)gates, (const T__*)x, (const T__*)w, (float*)pool, (const int*)state_in, (const int*)state_out, \
                     (const int*)seg, (const int*)seg_offsets, (const float*)a_log, (const float*)dt_bias, T_, H, G, dk, dkp, dv, taps,  \
                     x_stride, out_stride, b_off, a_off, q_scale, unit_eps
#define CD_LAUNCH(T__)                                                                                                              \
    do {                                                                                                                            \
        if (vec && wide) conv_delta_inputs_kernel<8, T__, 1024><<<cp_blocks(T_), 1024, nqk * 4, stream>>>(CD_ARGS(T__));            \
        else if (vec) conv_delta_inputs_kernel<8, T__, 256><<<cp_blocks(T_), 256, nqk * 4, stream>>>(CD_ARGS(T__));                 \
        else conv_delta_inputs_kernel<1, T__, 256><<<cp_blocks(T_), 256, nqk * 4, stream>>>(CD_ARGS(T__));                          \
    } while (0)
        if (dtype == ILM_DTYPE_F32) CD_LAUNCH(float);
        else if (dtype == ILM_DTYPE_BF16) CD_LAUNCH(bf16);
        else ILM_REQUIRE(false, "conv_delta_inputs: unknown dtype %d", dtype);
#undef CD_LAUNCH
#undef CD_ARGS
    }
    ILM_LAUNCH_CHECK("conv_delta_inputs");
    if (taps > 1 && !singles)
        return dtype == ILM_DTYPE_F32 ? cp_state<float>(x, pool, state_in, state_out, seg_offsets, R, C, taps, x_stride, stream)
                                      : cp_state<bf16>(x, pool, state_in, state_out, seg_offsets, R, C, taps, x_stride, stream);
    return 0;
}

// ------------------------------------------------------------------------------------------
// LDS floats: rows y [C] | cosines, sines [rd / 2 each]
template <int VEC, typename T, int THREADS, int MT>
__global__ void __launch_bounds__(THREADS, MT <= 4 && VEC == 8 ? 8 : 1)     // (up to 4 taps: 64 registers, as many waves as a unit holds)
conv_norm_rope_kvwrite_kernel(T* __restrict__ q_out, const T* __restrict__ x, const T* __restrict__ w, float* __restrict__ pool,
                              const int* __restrict__ state_in, const int* __restrict__ state_out, const int* __restrict__ seg,
                              const int* __restrict__ seg_offsets, const int* __restrict__ pos, const float* __restrict__ freq,
                              const T* __restrict__ wq, const T* __restrict__ wk, T* __restrict__ kc, T* __restrict__ vc,
                              const int* __restrict__ slots, int T_, int H, int G, int dim, int vdim, int d, int rd, int own_kv, int taps,
                              int x_stride, float eps, int page) {
    extern __shared__ __attribute__((aligned(16))) float sm[];
    __shared__ float red[2 * (THREADS / 64)];
    const int t = cp_token(T_);
    if (t < 0) return;
    const int tid = threadIdx.x;
    const int Cq = H * dim, Ck = own_kv ? G * dim : 0, C = Cq + Ck + (own_kv ? G * vdim : 0);
    float* cs = sm + (C + 3) / 4 * 4;
    const int half = rd >> 1;
    const cp_place p = cp_find(t, seg, seg_offsets, state_in, state_out, pool, taps, C);
    float sq = 0.f, sk = 0.f;
    for (int c = tid * VEC; c < C; c += THREADS * VEC) {
        float y[VEC];
        cp_conv<VEC, T, MT>(y, x, x_stride, w, t, c, C, taps, p);
        float s = 0.f;
        cp_store<VEC, float>(sm + c, y);
#pragma unroll
        for (int e = 0; e < VEC; ++e) s = fmaf(y[e], y[e], s);
        if (c < Cq) sq += s;
        else if (c < Cq + Ck) sk += s;
    }
    const float ps = (float)pos[t];
    for (int i = tid; i < half; i += THREADS) {
        float sn, cn;
        sincosf(ps * freq[i], &sn, &cn);
        cs[i] = cn;
        cs[half + i] = sn;
    }
    // both sums over the block's waves (the barrier also publishes sm and cs)
    sq = wave_sum(sq);
    sk = wave_sum(sk);
    if ((tid & 63) == 0) {
        red[tid >> 6] = sq;
        red[THREADS / 64 + (tid >> 6)] = sk;
    }
    __syncthreads();
    sq = sk = 0.f;
#pragma unroll
    for (int i = 0; i < THREADS / 64; ++i) {
        sq += red[i];
        sk += red[THREADS / 64 + i];
    }
    const float rq = wq != nullptr ? 1.0f / sqrtf(sq / (float)Cq + eps) : 1.0f;
    const float rk = wk != nullptr && own_kv ? 1.0f / sqrtf(sk / (float)Ck + eps) : 1.0f;
    const int slot = (own_kv && slots != nullptr) ? slots[t] : -1;
    const int pg = slot >= 0 ? slot / page : 0, off = slot >= 0 ? slot % page : 0;
    // pieces of 8 entries of q and k heads (of d entries in what is written; d is a multiple of 8)
    const int per = d >> 3, nq = H * per, nk = slot >= 0 ? G * per : 0;
    for (int it = tid; it < nq + nk; it += THREADS) {
        const bool is_q = it < nq;
        const int u = (is_q ? it : it - nq) / per, e0 = ((is_q ? it : it - nq) % per) * 8;
        const int src = (is_q ? 0 : Cq) + u * dim + e0;
        const T* wn = is_q ? wq : wk;
        const float f = is_q ? rq : rk;
        float v[8];
        if constexpr (VEC == 8) {        // (a piece lies inside its head whole, or beyond it whole)
            cp_load<8, float>(sm + (e0 < dim ? src : 0), v);
#pragma unroll
            for (int e = 0; e < 8; ++e) v[e] = e0 < dim ? v[e] * f : 0.f;
        } else {
#pragma unroll
            for (int e = 0; e < 8; ++e) v[e] = e0 + e < dim ? sm[src + e] * f : 0.f;
        }
        if (wn != nullptr) {
            if constexpr (VEC == 8) {
                if (e0 < dim) {
                    float wv[8];
                    cp_load<8, T>(wn + u * dim + e0, wv);
#pragma unroll
                    for (int e = 0; e < 8; ++e) v[e] *= wv[e];
                }
            } else {
#pragma unroll
                for (int e = 0; e < 8; ++e)
                    if (e0 + e < dim) v[e] *= to_f32(wn[u * dim + e0 + e]);
            }
        }
#pragma unroll
        for (int e = 0; e < 8; e += 2)
            if (e0 + e < rd) {
                const float c0 = cs[(e0 + e) >> 1], s0 = cs[half + ((e0 + e) >> 1)];
                const float a = v[e], b = v[e + 1];
                v[e] = a * c0 - b * s0;
                v[e + 1] = b * c0 + a * s0;
            }
        T* dst = is_q ? q_out + ((size_t)t * H + u) * d + e0 : kc + (((size_t)pg * G + u) * page + off) * d + e0;
        cp_store<8, T>(dst, v);
    }
    if (slot >= 0)
        for (int it = tid; it < G * vdim; it += THREADS)
            vc[((size_t)pg * G + it / vdim) * d * page + (size_t)(it % vdim) * page + off] = from_f32<T>(sm[Cq + Ck + it]);
}

extern "C" int ilm_conv_norm_rope_kvwrite(void* q_out, const void* x, const void* w, void* pool, const void* state_in,
                                          const void* state_out, const void* seg, const void* seg_offsets, const void* pos,
                                          const void* freq, const void* wq, const void* wk, void* kc, void* vc, const void* slots,
                                          int T_, int R, int H, int G, int dim, int vdim, int d, int rd, int own_kv, int taps,
                                          int x_stride, float eps, int page, int singles, int dtype, hipStream_t stream) {
    const int C = H * dim + (own_kv ? G * (dim + vdim) : 0);
    ILM_REQUIRE(T_ > 0 && R > 0 && R <= 65535 && H > 0 && G > 0 && dim > 0 && vdim > 0, "conv_norm_rope_kvwrite: bad sizes");
    ILM_REQUIRE(d % 8 == 0 && dim <= d && vdim <= d, "conv_norm_rope_kvwrite: heads of %d / %d in cache heads of %d", dim, vdim, d);
    ILM_REQUIRE(rd >= 0 && rd % 2 == 0 && rd <= dim && (rd == 0 || freq != nullptr), "conv_norm_rope_kvwrite: %d turned entries", rd);
    ILM_REQUIRE(taps >= 0 && taps <= CP_MAX_TAPS, "conv_norm_rope_kvwrite: %d taps, at most %d", taps, CP_MAX_TAPS);
    ILM_REQUIRE((taps <= 1 || pool != nullptr) && (taps == 0 || w != nullptr), "conv_norm_rope_kvwrite: a convolution needs its weights and state rows");
    ILM_REQUIRE(slots == nullptr || !own_kv || (kc != nullptr && vc != nullptr && page > 0), "conv_norm_rope_kvwrite: slots without a cache");
    ILM_REQUIRE(x_stride >= C, "conv_norm_rope_kvwrite: rows of %d elements are too short for %d", x_stride, C);
    ILM_REQUIRE((((uintptr_t)q_out | (uintptr_t)kc) & 15) == 0, "conv_norm_rope_kvwrite: results must be 16-byte aligned");
    const size_t shm = ((size_t)(C + 3) / 4 * 4 + rd) * sizeof(float);
    ILM_REQUIRE(shm <= CP_MAX_LDS, "conv_norm_rope_kvwrite: rows of %d channels do not fit LDS", C);
    const bool vec = dim % 8 == 0 && (own_kv ? (G * vdim) % 8 == 0 : true) && x_stride % 8 == 0
                     && (((uintptr_t)x | (uintptr_t)w | (uintptr_t)pool | (uintptr_t)wq | (uintptr_t)wk) & 15) == 0;
    const bool wide = T_ <= 2 * ilm_num_cus();
#define CN_ARGS(T__) (T__*)q_out, (const T__*)x, (const T__*)w, (float*)pool, (const int*)state_in, (const int*)state_out,            \
                     (const int*)seg, (const int*)seg_offsets, (const int*)pos, (const float*)freq, (const T__*)wq, (const T__*)wk,    \
                     (T__*)kc, (T__*)vc, (const int*)slots, T_, H, G, dim, vdim, d, rd, own_kv, taps, x_stride, eps, page
#define CN_LAUNCH_T(T__, MT_)                                                                                                       \
    do {                                                                                                                            \
        if (vec && wide) conv_norm_rope_kvwrite_kernel<8, T__, 1024, MT_><<<cp_blocks(T_), 1024, shm, stream>>>(CN_ARGS(T__));      \
        else if (vec) conv_norm_rope_kvwrite_kernel<8, T__, 256, MT_><<<cp_blocks(T_), 256, shm, stream>>>(CN_ARGS(T__));           \
        else conv_norm_rope_kvwrite_kernel<1, T__, 256, MT_><<<cp_blocks(T_), 256, shm, stream>>>(CN_ARGS(T__));                    \
    } while (0)
#define CN_LAUNCH(T__)                                       \
    do {                                                     \
        if (taps <= 4) CN_LAUNCH_T(T__, 4);                  \
        else CN_LAUNCH_T(T__, CP_MAX_TAPS);                  \
    } while (0)
    if (dtype == ILM_DTYPE_F32) CN_LAUNCH(float);
    else if (dtype == ILM_DTYPE_BF16) CN_LAUNCH(bf16);
    else ILM_REQUIRE(false, "conv_norm_rope_kvwrite: unknown dtype %d", dtype);
#undef CN_LAUNCH
#undef CN_LAUNCH_T
#undef CN_ARGS
    ILM_LAUNCH_CHECK("conv_norm_rope_kvwrite");
    if (taps > 1 && !singles)
        return dtype == ILM_DTYPE_F32 ? cp_state<float>(x, pool, state_in, state_out, seg_offsets, R, C, taps, x_stride, stream)
                                      : cp_state<bf16>(x, pool, state_in, state_out, seg_offsets, R, C, taps, x_stride, stream);
    return 0;
}
