//! `HipHybridRunner`: sequences and batched steps of the hybrid decoder (`crabml_hip_hybrid_*`) -- models whose layers mix
//! softmax attention (in chunks, in a window, on latents) with decaying linear attention, gated units and residual streams,
//! which crabml's `Tensor` trait has no op sequence for.  The caller
//! fills `crabml_hip_hybrid_config_t` / `_layer_t` / `_weights_t` from its model files; matrices are copied at creation, so the
//! tensors behind the handles may be dropped afterwards.

use std::ptr;

use crabml::error::Result;

pub use crate::ffi::crabml_hip_hybrid_config_t;
pub use crate::ffi::crabml_hip_hybrid_layer_t;
pub use crate::ffi::crabml_hip_hybrid_weights_t;

use crate::ffi;
use crate::HipTensorDeviceRef;

/// One sequence's part of a step: its next tokens, and the places among them whose logits are wanted (ascending).
pub struct StepEntry<'a> {
    pub seq: usize,
    pub tokens: &'a [u32],
    pub want: &'a [u32],
}

pub struct HipHybridRunner {
    raw: *mut ffi::crabml_hip_hybrid_t,
    vocab_size: usize,
    device: HipTensorDeviceRef,
}

unsafe impl Send for HipHybridRunner {}

impl HipHybridRunner {
    pub fn new(
        conf: &crabml_hip_hybrid_config_t,
        layers: &[crabml_hip_hybrid_layer_t],
        weights: &crabml_hip_hybrid_weights_t,
        device: HipTensorDeviceRef,
    ) -> Result<Self> {
        assert_eq!(conf.n_layers, layers.len());
        let mut raw = ptr::null_mut();
        device.check(unsafe {
            ffi::crabml_hip_hybrid_create(device.raw, conf, layers.as_ptr(), weights, &mut raw)
        })?;
        Ok(Self {
            raw,
            vocab_size: conf.vocab_size,
            device,
        })
    }

    pub fn open(&mut self) -> Result<usize> {
        let mut seq = 0usize;
        self.device
            .check(unsafe { ffi::crabml_hip_hybrid_open(self.raw, &mut seq) })?;
        Ok(seq)
    }

    /// gives the sequence's state back; the next one opened may get the same slab
    pub fn close(&mut self, seq: usize) -> Result<()> {
        self.device
            .check(unsafe { ffi::crabml_hip_hybrid_close(self.raw, seq) })
    }

    pub fn len(&self, seq: usize) -> usize {
        unsafe { ffi::crabml_hip_hybrid_len(self.raw, seq) }
    }

    /// One batch; returns the wanted logits, `vocab_size` numbers each, in the order of the entries and of their `want`.
    pub fn step(&mut self, entries: &[StepEntry]) -> Result<Vec<f32>> {
        let seqs = entries.iter().map(|e| e.seq).collect::<Vec<_>>();
        let counts = entries.iter().map(|e| e.tokens.len()).collect::<Vec<_>>();
        let want_counts = entries.iter().map(|e| e.want.len()).collect::<Vec<_>>();
        let tokens = entries.iter().flat_map(|e| e.tokens.iter().copied()).collect::<Vec<_>>();
        let want = entries.iter().flat_map(|e| e.want.iter().copied()).collect::<Vec<_>>();
        let mut logits = vec![0f32; want.len() * self.vocab_size];
        self.device.check(unsafe {
            ffi::crabml_hip_hybrid_step(
                self.raw,
                entries.len(),
                seqs.as_ptr(),
                counts.as_ptr(),
                tokens.as_ptr(),
                want_counts.as_ptr(),
                want.as_ptr(),
                logits.as_mut_ptr(),
            )
        })?;
        Ok(logits)
    }

    /// `steps` greedy steps of up to 16 sequences on the device; row s of the result holds step s's tokens.
    pub fn decode_greedy(&mut self, seqs: &[usize], tokens: &[u32], steps: usize) -> Result<Vec<u32>> {
        assert_eq!(seqs.len(), tokens.len());
        let mut out = vec![0u32; steps * seqs.len()];
        self.device.check(unsafe {
            ffi::crabml_hip_hybrid_decode_greedy(
                self.raw,
                seqs.len(),
                seqs.as_ptr(),
                tokens.as_ptr(),
                steps,
                out.as_mut_ptr(),
            )
        })?;
        Ok(out)
    }
}

impl Drop for HipHybridRunner {
    fn drop(&mut self) {
        unsafe { ffi::crabml_hip_hybrid_destroy(self.raw) };
    }
}
